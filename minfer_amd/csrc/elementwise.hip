// Row-wise and element-wise kernels: embedding gather, RMSNorm (with optional row
// gather), SwiGLU, rotation table, rotation fused with the cache write, type conversion,
// seeded normal fill.  Formulas follow yusiwen/minfer's CPU path; each kernel names its
// source.  Statistics, angles and the residual stream are 32-bit.
#include "common.h"
#include "random_normal.h"

// ---------------------------------------------------------------- embedding
// h[t][:] = table[ids[t]][:] (src/graph/cpu_backend.rs:269-285), times a scale where a design has
// one.  The host checks ids before upload; an id outside the table gives a row of NaN so that it shows.
template <typename TT>
__global__ __launch_bounds__(256) void embed_kernel(const TT* __restrict__ table,
                                                    const int* __restrict__ ids,
                                                    float* __restrict__ out, int d, int vocab, float scale) {
  const int row = blockIdx.x;
  const int id = ids[row];
  float* o = out + (size_t)row * d;
  if (id < 0 || id >= vocab) {
    for (int i = threadIdx.x; i < d; i += 256) o[i] = __builtin_nanf("");
    return;
  }
  const TT* src = table + (size_t)id * d;
  for (int i = threadIdx.x; i < d; i += 256) o[i] = to_f32(src[i]) * scale;
}

MF_API int mf_embed(const void* table, int table_is_bf16, const int* ids, float* out, int rows,
                    int d, int vocab, float scale, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (table_is_bf16)
    embed_kernel<bf16><<<rows, 256, 0, stream>>>((const bf16*)table, ids, out, d, vocab, scale);
  else
    embed_kernel<float><<<rows, 256, 0, stream>>>((const float*)table, ids, out, d, vocab, scale);
  return mf_launch_status();
}

// ---------------------------------------------------------------- table row + row of the pair with the token before
// out[t][:] = table[ids[t]][:] scale + pairs[row][:], row = (previous mul_prev + id mul_cur) mod buckets, and row
// `buckets` for a sequence's first token.  The previous token is the one ahead in the step, or, for the first token a
// sequence brings, its state `last[slot]`; the workgroup of that token also leaves the sequence's last token there, so
// that one workgroup reads and writes a slot's state.  An id outside the table gives a row of NaN, as `embed_kernel` does.
template <typename TT>
__global__ __launch_bounds__(256) void embed_pairs_kernel(const TT* __restrict__ table, const TT* __restrict__ pairs,
                                                          const int* __restrict__ ids, const int* __restrict__ positions,
                                                          const int* __restrict__ seq_of_tok,
                                                          const int* __restrict__ cu_seqlens,
                                                          const int* __restrict__ slot_ids, int* __restrict__ last,
                                                          float* __restrict__ out, int d, int vocab, int buckets,
                                                          long long mul_prev, long long mul_cur, float scale) {
  __shared__ int row_of;
  const int t = blockIdx.x;
  if (threadIdx.x == 0) {
    const int b = seq_of_tok[t], first = cu_seqlens[b];
    int before = t > first ? ids[t - 1] : -1;
    if (t == first) {
      int* mine = last + slot_ids[b];
      if (positions[t] > 0) before = *mine;
      *mine = ids[cu_seqlens[b + 1] - 1];
    }
    const long long sum = (long long)before * mul_prev + (long long)ids[t] * mul_cur;
    row_of = positions[t] > 0 ? (int)((sum % buckets + buckets) % buckets) : buckets;
  }
  __syncthreads();
  const int id = ids[t];
  float* o = out + (size_t)t * d;
  if (id < 0 || id >= vocab) {
    for (int i = threadIdx.x; i < d; i += 256) o[i] = __builtin_nanf("");
    return;
  }
  const TT* src = table + (size_t)id * d;
  const TT* pr = pairs + (size_t)row_of * d;
  for (int i = threadIdx.x; i < d; i += 256) o[i] = fmaf(to_f32(src[i]), scale, to_f32(pr[i]));
}

// table [vocab][d], pairs [buckets + 1][d] of one type; last int32 [slots]
MF_API int mf_embed_pairs(const void* table, const void* pairs, int tables_are_bf16, const int* ids, const int* positions,
                          const int* seq_of_tok, const int* cu_seqlens, const int* slot_ids, int* last, float* out, int rows,
                          int d, int vocab, int buckets, long long mul_prev, long long mul_cur, float scale,
                          hipStream_t stream) {
  if (rows <= 0) return 0;
  if (d <= 0 || vocab <= 0 || buckets <= 0) return (int)hipErrorInvalidValue;
  if (tables_are_bf16)
    embed_pairs_kernel<bf16><<<rows, 256, 0, stream>>>((const bf16*)table, (const bf16*)pairs, ids, positions, seq_of_tok,
                                                        cu_seqlens, slot_ids, last, out, d, vocab, buckets, mul_prev, mul_cur,
                                                        scale);
  else
    embed_pairs_kernel<float><<<rows, 256, 0, stream>>>((const float*)table, (const float*)pairs, ids, positions, seq_of_tok,
                                                         cu_seqlens, slot_ids, last, out, d, vocab, buckets, mul_prev, mul_cur,
                                                         scale);
  return mf_launch_status();
}

// ---------------------------------------------------------------- RMSNorm
// y = x * (1/sqrt(mean(x^2) + eps)) * w  (src/vec_ops.rs:500-522; eps inside the root).
// Row r of the output reads row row_idx[r] of x when row_idx is given.
// A row of at most 256 * 4 * KEEP elements stays in registers between the sum and the scaling.
template <typename OT, int KEEP>
__device__ __forceinline__ void rmsnorm_row_kept(const float* __restrict__ xr, const float* __restrict__ w,
                                                 OT* __restrict__ o, int d, float eps, float* scratch) {
  float4 v[KEEP];
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < KEEP; ++c) {
    const int i = (c * 256 + threadIdx.x) * 4;
    v[c] = i < d ? *reinterpret_cast<const float4*>(xr + i) : make_float4(0.f, 0.f, 0.f, 0.f);
    ss = fmaf(v[c].x, v[c].x, ss);
    ss = fmaf(v[c].y, v[c].y, ss);
    ss = fmaf(v[c].z, v[c].z, ss);
    ss = fmaf(v[c].w, v[c].w, ss);
  }
  ss = block_sum<256>(ss, scratch);
  const float scale = 1.0f / sqrtf(ss / (float)d + eps);
#pragma unroll
  for (int c = 0; c < KEEP; ++c) {
    const int i = (c * 256 + threadIdx.x) * 4;
    if (i < d) {
      const float4 g = w ? *reinterpret_cast<const float4*>(w + i) : make_float4(1.f, 1.f, 1.f, 1.f);
      o[i + 0] = from_f32<OT>(v[c].x * scale * g.x);
      o[i + 1] = from_f32<OT>(v[c].y * scale * g.y);
      o[i + 2] = from_f32<OT>(v[c].z * scale * g.z);
      o[i + 3] = from_f32<OT>(v[c].w * scale * g.w);
    }
  }
}

template <typename OT>
__global__ __launch_bounds__(256) void rmsnorm_kernel(const float* __restrict__ x,
                                                      const int* __restrict__ row_idx,
                                                      const float* __restrict__ w,
                                                      OT* __restrict__ out, int d, float eps, int ld) {
  __shared__ float scratch[4];
  const int row = blockIdx.x;
  const float* xr = x + (size_t)(row_idx ? row_idx[row] : row) * ld;      // (ld > d: the first d values of longer rows)
  OT* o = out + (size_t)row * d;
  if (d % 4 == 0 && ld % 4 == 0 && d <= 256 * 4 * 16) {
    if (d <= 256 * 4 * 4) rmsnorm_row_kept<OT, 4>(xr, w, o, d, eps, scratch);
    else if (d <= 256 * 4 * 8) rmsnorm_row_kept<OT, 8>(xr, w, o, d, eps, scratch);
    else rmsnorm_row_kept<OT, 16>(xr, w, o, d, eps, scratch);
    return;
  }
  float ss = 0.f;
  for (int i = threadIdx.x; i < d; i += 256) {
    const float v = xr[i];
    ss = fmaf(v, v, ss);
  }
  ss = block_sum<256>(ss, scratch);
  const float scale = 1.0f / sqrtf(ss / (float)d + eps);
  for (int i = threadIdx.x; i < d; i += 256) {
    const float g = w ? w[i] : 1.0f;
    o[i] = from_f32<OT>(xr[i] * scale * g);
  }
}

MF_API int mf_rmsnorm(const float* x, const int* row_idx, const float* w, void* out,
                      int out_is_bf16, int rows, int d, float eps, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (out_is_bf16)
    rmsnorm_kernel<bf16><<<rows, 256, 0, stream>>>(x, row_idx, w, (bf16*)out, d, eps, d);
  else
    rmsnorm_kernel<float><<<rows, 256, 0, stream>>>(x, row_idx, w, (float*)out, d, eps, d);
  return mf_launch_status();
}

// the norm over the first d values of rows of ld values
MF_API int mf_rmsnorm_cols(const float* x, int ld, const float* w, void* out, int out_is_bf16, int rows, int d, float eps,
                           hipStream_t stream) {
  if (rows <= 0) return 0;
  if (d < 1 || ld < d) return (int)hipErrorInvalidValue;
  if (out_is_bf16)
    rmsnorm_kernel<bf16><<<rows, 256, 0, stream>>>(x, nullptr, w, (bf16*)out, d, eps, ld);
  else
    rmsnorm_kernel<float><<<rows, 256, 0, stream>>>(x, nullptr, w, (float*)out, d, eps, ld);
  return mf_launch_status();
}

// ---------------------------------------------------------------- RMS norm in groups
// The row is cut into `groups` equal consecutive parts; each part is divided by its own
// sqrt(mean(part^2) + eps) and the whole is multiplied by w.  Three uses of one kernel:
// write the normed row (run type), add it into a 32-bit row (a residual stream that takes a
// branch's normed output: h += N(y)), and, with the sum, leave the new row rounded to bfloat16
// as well for the product that reads the stream next.  x and out may be the same rows (a part is
// summed before any of it is written).
template <typename OT, bool ADD>
__global__ __launch_bounds__(256) void group_rmsnorm_kernel(const float* x,
                                                            const int* __restrict__ row_idx,
                                                            const float* __restrict__ w, OT* out,
                                                            bf16* __restrict__ cast_out, int d, int groups,
                                                            float eps) {
  __shared__ float scratch[4];
  const int row = blockIdx.x;
  const float* xr = x + (size_t)(row_idx ? row_idx[row] : row) * d;
  OT* o = out + (size_t)row * d;
  bf16* co = cast_out ? cast_out + (size_t)row * d : nullptr;
  const int part = d / groups;
  // a number of groups that is a power of two up to 256: every group has 256 / groups threads of its
  // own and all groups go at once (a row's loads are all in flight together); else group by group
  if ((groups & (groups - 1)) == 0 && groups <= 256) {
    const int tpg = 256 / groups;                  // threads of a group: a power of two
    const int g = threadIdx.x / tpg, tl = threadIdx.x % tpg;
    const int lo = g * part;
    auto group_total = [&](float ss) {
#pragma unroll
      for (int off = 1; off < 64; off <<= 1)
        if (off < tpg) ss += __shfl_xor(ss, off, MF_WAVE);
      if (tpg > 64) {                              // the group's waves meet in LDS
        const int wv = threadIdx.x >> 6;
        if ((threadIdx.x & 63) == 0) scratch[wv] = ss;
        __syncthreads();
        const int w0 = (wv / (tpg / 64)) * (tpg / 64);
        ss = 0.f;
        for (int k = 0; k < tpg / 64; ++k) ss += scratch[w0 + k];
      }
      return ss;
    };
    constexpr int KEEP = 16;
    if (d % 256 == 0 && d <= 256 * KEEP) {         // a thread's d / 256 values, gains and old sums in one trip
      const int ept = d / 256;
      float xv[KEEP], gv[KEEP], ov[KEEP];
      float ss = 0.f;
#pragma unroll
      for (int k = 0; k < KEEP; ++k) {
        const int i = lo + tl + k * tpg;
        xv[k] = k < ept ? xr[i] : 0.f;
        gv[k] = (k < ept && w) ? w[i] : 1.0f;
        ov[k] = (ADD && k < ept) ? to_f32(o[i]) : 0.f;
        ss = fmaf(xv[k], xv[k], ss);
      }
      const float scale = 1.0f / sqrtf(group_total(ss) / (float)part + eps);
#pragma unroll
      for (int k = 0; k < KEEP; ++k) {
        if (k < ept) {
          const int i = lo + tl + k * tpg;
          const float y = xv[k] * scale * gv[k] + ov[k];
          o[i] = from_f32<OT>(y);
          if (co) co[i] = (bf16)y;
        }
      }
      return;
    }
    float ss = 0.f;
    for (int i = tl; i < part; i += tpg) {
      const float v = xr[lo + i];
      ss = fmaf(v, v, ss);
    }
    const float scale = 1.0f / sqrtf(group_total(ss) / (float)part + eps);
    for (int i = tl; i < part; i += tpg) {
      float y = xr[lo + i] * scale * (w ? w[lo + i] : 1.0f);
      if (ADD) y += to_f32(o[lo + i]);
      o[lo + i] = from_f32<OT>(y);
      if (co) co[lo + i] = (bf16)y;
    }
    return;
  }
  for (int g = 0; g < groups; ++g) {
    const int lo = g * part;
    float ss = 0.f;
    for (int i = threadIdx.x; i < part; i += 256) {
      const float v = xr[lo + i];
      ss = fmaf(v, v, ss);
    }
    ss = block_sum<256>(ss, scratch);
    const float scale = 1.0f / sqrtf(ss / (float)part + eps);
    for (int i = threadIdx.x; i < part; i += 256) {
      float y = xr[lo + i] * scale * (w ? w[lo + i] : 1.0f);
      if (ADD) y += to_f32(o[lo + i]);
      o[lo + i] = from_f32<OT>(y);
      if (co) co[lo + i] = (bf16)y;
    }
    __syncthreads();
  }
}

MF_API int mf_group_rmsnorm(const float* x, const int* row_idx, const float* w, void* out, int out_is_bf16,
                            int add, void* cast_out, int rows, int d, int groups, float eps,
                            hipStream_t stream) {
  if (rows <= 0) return 0;
  if (groups < 1 || d % groups != 0 || (add && out_is_bf16)) return (int)hipErrorInvalidValue;
  if (add)
    group_rmsnorm_kernel<float, true><<<rows, 256, 0, stream>>>(x, row_idx, w, (float*)out, (bf16*)cast_out, d,
                                                                 groups, eps);
  else if (out_is_bf16)
    group_rmsnorm_kernel<bf16, false><<<rows, 256, 0, stream>>>(x, row_idx, w, (bf16*)out, (bf16*)cast_out, d,
                                                                 groups, eps);
  else
    group_rmsnorm_kernel<float, false><<<rows, 256, 0, stream>>>(x, row_idx, w, (float*)out, (bf16*)cast_out, d,
                                                                  groups, eps);
  return mf_launch_status();
}

// ---------------------------------------------------------------- xIELU
// z > 0: a_pos z^2 + z/2;  z <= 0: a_neg (e^z - 1 - z) + z/2, where a_pos = softplus(p) and
// a_neg = 1/2 + softplus(q) come from the layer's two learned numbers (the host works them out).
__device__ __forceinline__ float xielu_of(float z, float a_pos, float a_neg) {
  return z > 0.f ? fmaf(a_pos * z, z, 0.5f * z) : fmaf(a_neg, expm1f(z) - z, 0.5f * z);
}

template <typename OT>
__global__ __launch_bounds__(256) void xielu_kernel(const float* __restrict__ x, OT* __restrict__ out, size_t n,
                                                    float a_pos, float a_neg) {
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i < n) out[i] = from_f32<OT>(xielu_of(x[i], a_pos, a_neg));
}

MF_API int mf_xielu(const float* x, void* out, int out_is_bf16, size_t n, float a_pos, float a_neg,
                    hipStream_t stream) {
  if (n == 0) return 0;
  const unsigned blocks = (unsigned)((n + 255) / 256);
  if (out_is_bf16)
    xielu_kernel<bf16><<<blocks, 256, 0, stream>>>(x, (bf16*)out, n, a_pos, a_neg);
  else
    xielu_kernel<float><<<blocks, 256, 0, stream>>>(x, (float*)out, n, a_pos, a_neg);
  return mf_launch_status();
}

// out[r][:] = x[idx[r]][:]  (generic row selection, src/graph/cpu_backend.rs:255-268)
__global__ __launch_bounds__(256) void gather_rows_kernel(const float* __restrict__ x,
                                                          const int* __restrict__ idx,
                                                          float* __restrict__ out, int d) {
  const float* src = x + (size_t)idx[blockIdx.x] * d;
  float* o = out + (size_t)blockIdx.x * d;
  for (int i = threadIdx.x; i < d; i += 256) o[i] = src[i];
}

MF_API int mf_gather_rows(const float* x, const int* idx, float* out, int rows, int d,
                          hipStream_t stream) {
  if (rows <= 0) return 0;
  gather_rows_kernel<<<rows, 256, 0, stream>>>(x, idx, out, d);
  return mf_launch_status();
}

// ---------------------------------------------------------------- SwiGLU
// y[r][i] = silu(g[r][i]) * u[r][i], silu(z) = z / (1 + exp(-z))
// (src/vec_ops.rs:131-146, src/graph/cpu_backend.rs:323-329).  g and u are the two halves
// of one [rows][2*nf] buffer.
template <typename IT, typename OT>
__global__ __launch_bounds__(256) void swiglu_kernel(const IT* __restrict__ gu, OT* __restrict__ out,
                                                     int nf, float limit) {
  const IT* g = gu + (size_t)blockIdx.y * 2 * nf;
  const IT* u = g + nf;
  OT* o = out + (size_t)blockIdx.y * nf;
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i < nf) {
    const float z = to_f32(g[i]);
    o[i] = from_f32<OT>(limit > 0.f ? clamped_gate(z, to_f32(u[i]), limit) : z / (1.0f + expf(-z)) * to_f32(u[i]));
  }
}

// limit > 0: the clamped form, g = min(gate, limit), u = clamp(up, -limit, limit), g sigmoid(1.702 g) (u + 1)
MF_API int mf_swiglu(const void* gu, int in_is_bf16, void* out, int out_is_bf16, int rows, int nf, float limit,
                     hipStream_t stream) {
  if (rows <= 0) return 0;
  dim3 grid((nf + 255) / 256, rows);
  if (in_is_bf16 && out_is_bf16)
    swiglu_kernel<bf16, bf16><<<grid, 256, 0, stream>>>((const bf16*)gu, (bf16*)out, nf, limit);
  else if (!in_is_bf16 && out_is_bf16)
    swiglu_kernel<float, bf16><<<grid, 256, 0, stream>>>((const float*)gu, (bf16*)out, nf, limit);
  else if (!in_is_bf16 && !out_is_bf16)
    swiglu_kernel<float, float><<<grid, 256, 0, stream>>>((const float*)gu, (float*)out, nf, limit);
  else
    return (int)hipErrorInvalidValue;
  return mf_launch_status();
}

// ---------------------------------------------------------------- type conversion
template <typename IT, typename OT>
__global__ __launch_bounds__(256) void convert_kernel(const IT* __restrict__ in, OT* __restrict__ out,
                                                      size_t n) {
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256)
    out[i] = from_f32<OT>(to_f32(in[i]));
}

MF_API int mf_convert(const void* in, int in_is_bf16, void* out, int out_is_bf16, size_t n,
                      hipStream_t stream) {
  if (n == 0) return 0;
  const int blocks = (int)((n + 255) / 256 < 65535 ? (n + 255) / 256 : 65535);
  if (in_is_bf16 && !out_is_bf16)
    convert_kernel<bf16, float><<<blocks, 256, 0, stream>>>((const bf16*)in, (float*)out, n);
  else if (!in_is_bf16 && out_is_bf16)
    convert_kernel<float, bf16><<<blocks, 256, 0, stream>>>((const float*)in, (bf16*)out, n);
  else
    return (int)hipErrorInvalidValue;
  return mf_launch_status();
}

// ---------------------------------------------------------------- rotation
// cos/sin[pos][i] of angle = pos * scale / theta^(2i/hd), computed in double and rounded
// once (the reference forms the same angle in f32 per element and call,
// src/graph/cpu_backend.rs:403-420).
__global__ __launch_bounds__(256) void rope_table_kernel(float* __restrict__ cs, float* __restrict__ sn,
                                                         int n_pos, int half, double theta,
                                                         double freq_scale) {
  const int idx = blockIdx.x * 256 + threadIdx.x;
  if (idx >= n_pos * half) return;
  const int pos = idx / half, i = idx % half;
  const double freq = freq_scale / pow(theta, (2.0 * i) / (2.0 * half));
  const double ang = (double)pos * freq;
  cs[idx] = (float)cos(ang);
  sn[idx] = (float)sin(ang);
}

MF_API int mf_rope_table(float* cs, float* sn, int n_pos, int half, double theta,
                         double freq_scale, hipStream_t stream) {
  const int n = n_pos * half;
  if (n <= 0) return 0;
  rope_table_kernel<<<(n + 255) / 256, 256, 0, stream>>>(cs, sn, n_pos, half, theta, freq_scale);
  return mf_launch_status();
}

// cos and sin of position * freq[i], times `magnitude`, for frequencies the host has worked out
// in double (any ladder: plain, blended towards longer periods, ...): [n_pos][half].
__global__ __launch_bounds__(256) void rope_table_freqs_kernel(float* __restrict__ cs, float* __restrict__ sn,
                                                               const double* __restrict__ freqs, int n_pos,
                                                               int half, double magnitude) {
  const int idx = blockIdx.x * 256 + threadIdx.x;
  if (idx >= n_pos * half) return;
  const int pos = idx / half, i = idx % half;
  const double ang = (double)pos * freqs[i];
  cs[idx] = (float)(cos(ang) * magnitude);
  sn[idx] = (float)(sin(ang) * magnitude);
}

MF_API int mf_rope_table_freqs(float* cs, float* sn, const double* freqs, int n_pos, int half,
                               double magnitude, hipStream_t stream) {
  const int n = n_pos * half;
  if (n <= 0) return 0;
  rope_table_freqs_kernel<<<(n + 255) / 256, 256, 0, stream>>>(cs, sn, freqs, n_pos, half, magnitude);
  return mf_launch_status();
}

// Half-split rotation of q and k (pair i with i + hd/2; x0' = x0 c - x1 s, x1' = x0 s + x1 c;
// src/graph/cpu_backend.rs:421-431), v copied, k and v stored into the paged cache at the
// token's position before attention reads it (src/graph/cpu_backend.rs:118-149).  Without
// tables (cs null) nothing is rotated: the kernel then only rounds q and stores k and v that
// some other position encoding has already treated.
// qkv is [T][(nh + 2 nk) hd] in 32-bit with biases already added.  One block per
// (token, head of q|k|v).
// In bfloat16 a page of V is stored transposed in two halves, [2][hd][32 keys], the layout the
// attention kernels read as a matrix-core operand; in 32-bit it lies like K, [64 keys][hd].
template <typename OT, bool V_TRANSPOSED>
__global__ __launch_bounds__(64) void rope_kvwrite_kernel(
    const float* __restrict__ qkv, const float* __restrict__ cs, const float* __restrict__ sn,
    const int* __restrict__ positions, const int* __restrict__ seq_of_tok,
    const int* __restrict__ page_table, int pt_stride, OT* __restrict__ q_out,
    OT* __restrict__ kcache, OT* __restrict__ vcache, int nh, int nk, int hd, int write_kv) {
  const int t = blockIdx.x, head = blockIdx.y;
  const int half = hd >> 1;
  const int pos = positions[t];
  const float* src = qkv + ((size_t)t * (nh + 2 * nk) + head) * hd;
  if (head < nh) {
    OT* dst = q_out + ((size_t)t * nh + head) * hd;
    for (int i = threadIdx.x; i < half; i += 64) {
      const float c = cs ? cs[(size_t)pos * half + i] : 1.f, s = cs ? sn[(size_t)pos * half + i] : 0.f;
      const float x0 = src[i], x1 = src[i + half];
      dst[i] = from_f32<OT>(x0 * c - x1 * s);
      dst[i + half] = from_f32<OT>(x0 * s + x1 * c);
    }
    return;
  }
  if (!write_kv) return;
  const int page = page_table[(size_t)seq_of_tok[t] * pt_stride + pos / MF_PAGE];
  if (page < 0) return;
  const bool is_k = head < nh + nk;
  const int hk = is_k ? head - nh : head - nh - nk;
  if (is_k) {
    OT* dst = kcache + (((size_t)page * nk + hk) * MF_PAGE + pos % MF_PAGE) * hd;
    for (int i = threadIdx.x; i < half; i += 64) {
      const float c = cs ? cs[(size_t)pos * half + i] : 1.f, s = cs ? sn[(size_t)pos * half + i] : 0.f;
      const float x0 = src[i], x1 = src[i + half];
      dst[i] = from_f32<OT>(x0 * c - x1 * s);
      dst[i + half] = from_f32<OT>(x0 * s + x1 * c);
    }
  } else if (V_TRANSPOSED) {      // a page of V is [2][hd][32 keys]
    constexpr int VH = MF_PAGE / 2;
    const int off = pos % MF_PAGE;
    OT* dst = vcache + (((size_t)page * nk + hk) * 2 + off / VH) * hd * VH + off % VH;
    for (int i = threadIdx.x; i < hd; i += 64) dst[(size_t)i * VH] = from_f32<OT>(src[i]);
  } else {
    OT* dst = vcache + (((size_t)page * nk + hk) * MF_PAGE + pos % MF_PAGE) * hd;
    for (int i = threadIdx.x; i < hd; i += 64) dst[i] = from_f32<OT>(src[i]);
  }
}

// The same for head sizes that are multiples of 8 and 16-byte aligned rows: one block per token,
// a thread takes four neighbouring pairs at a time (float4 loads of x, cos and sin, one 8- or
// 16-byte store per half), q and k heads first, then v: the same bytes as one wave per token and
// head with 4-byte accesses moves, in wide accesses.
template <typename OT>
__device__ __forceinline__ void store4(OT* dst, float a, float b, float c, float d);
template <>
__device__ __forceinline__ void store4<float>(float* dst, float a, float b, float c, float d) {
  *reinterpret_cast<float4*>(dst) = make_float4(a, b, c, d);
}
template <>
__device__ __forceinline__ void store4<bf16>(bf16* dst, float a, float b, float c, float d) {
  *reinterpret_cast<bf16x4*>(dst) = bf16x4{(bf16)a, (bf16)b, (bf16)c, (bf16)d};
}

template <typename OT, bool V_TRANSPOSED>
__global__ __launch_bounds__(256) void rope_kvwrite_vec_kernel(
    const float* __restrict__ qkv, const float* __restrict__ cs, const float* __restrict__ sn,
    const int* __restrict__ positions, const int* __restrict__ seq_of_tok,
    const int* __restrict__ page_table, int pt_stride, OT* __restrict__ q_out,
    OT* __restrict__ kcache, OT* __restrict__ vcache, int nh, int nk, int hd, int write_kv) {
  const int t = blockIdx.x;
  const int half = hd >> 1, groups = half >> 2;           // groups of four pairs per head
  const int pos = positions[t];
  const float* row = qkv + (size_t)t * (nh + 2 * nk) * hd;
  const int page = write_kv ? page_table[(size_t)seq_of_tok[t] * pt_stride + pos / MF_PAGE] : -1;
  const int off = pos % MF_PAGE;
  const int n_rot = (nh + (write_kv && page >= 0 ? nk : 0)) * groups;
  for (int it = threadIdx.x; it < n_rot; it += 256) {
    const int head = it / groups, i = (it % groups) * 4;
    const float* src = row + (size_t)head * hd;
    const float4 x0 = *reinterpret_cast<const float4*>(src + i);
    const float4 x1 = *reinterpret_cast<const float4*>(src + i + half);
    const float4 c = cs ? *reinterpret_cast<const float4*>(cs + (size_t)pos * half + i) : make_float4(1.f, 1.f, 1.f, 1.f);
    const float4 s = cs ? *reinterpret_cast<const float4*>(sn + (size_t)pos * half + i) : make_float4(0.f, 0.f, 0.f, 0.f);
    OT* dst = head < nh ? q_out + ((size_t)t * nh + head) * hd
                        : kcache + (((size_t)page * nk + (head - nh)) * MF_PAGE + off) * hd;
    store4<OT>(dst + i, x0.x * c.x - x1.x * s.x, x0.y * c.y - x1.y * s.y, x0.z * c.z - x1.z * s.z,
               x0.w * c.w - x1.w * s.w);
    store4<OT>(dst + i + half, x0.x * s.x + x1.x * c.x, x0.y * s.y + x1.y * c.y, x0.z * s.z + x1.z * c.z,
               x0.w * s.w + x1.w * c.w);
  }
  if (!write_kv || page < 0) return;
  const float* vsrc = row + (size_t)(nh + nk) * hd;
  for (int it = threadIdx.x; it < nk * (hd >> 2); it += 256) {
    const int hk = it / (hd >> 2), i = (it % (hd >> 2)) * 4;
    const float4 v = *reinterpret_cast<const float4*>(vsrc + (size_t)hk * hd + i);
    if (V_TRANSPOSED) {                   // a page of V is [2][hd][32 keys]
      constexpr int VH = MF_PAGE / 2;
      OT* dst = vcache + ((((size_t)page * nk + hk) * 2 + off / VH) * hd + i) * VH + off % VH;
      dst[0] = from_f32<OT>(v.x);
      dst[VH] = from_f32<OT>(v.y);
      dst[2 * VH] = from_f32<OT>(v.z);
      dst[3 * VH] = from_f32<OT>(v.w);
    } else {
      store4<OT>(vcache + (((size_t)page * nk + hk) * MF_PAGE + off) * hd + i, v.x, v.y, v.z, v.w);
    }
  }
}

// The rotation alone, in place, on the first n_rot heads of every token's [n_heads_total][hd] row
// of 32-bit values (q and k of a q|k|v row; v is left as it is).
__global__ __launch_bounds__(256) void rope_inplace_kernel(float* __restrict__ x, const float* __restrict__ cs,
                                                           const float* __restrict__ sn,
                                                           const int* __restrict__ positions, int n_rot,
                                                           int n_heads_total, int hd) {
  const int t = blockIdx.x, half = hd >> 1;
  const int pos = positions[t];
  float* row = x + (size_t)t * n_heads_total * hd;
  for (int it = threadIdx.x; it < n_rot * half; it += 256) {
    const int head = it / half, i = it % half;
    const float c = cs[(size_t)pos * half + i], s = sn[(size_t)pos * half + i];
    float* p = row + (size_t)head * hd;
    const float x0 = p[i], x1 = p[i + half];
    p[i] = x0 * c - x1 * s;
    p[i + half] = x0 * s + x1 * c;
  }
}

MF_API int mf_rope_inplace(float* x, const float* cs, const float* sn, const int* positions, int n_tok, int n_rot,
                           int n_heads_total, int hd, hipStream_t stream) {
  if (n_tok <= 0 || n_rot <= 0) return 0;
  if (hd % 2 != 0 || n_rot > n_heads_total || !cs || !sn) return (int)hipErrorInvalidValue;
  rope_inplace_kernel<<<n_tok, 256, 0, stream>>>(x, cs, sn, positions, n_rot, n_heads_total, hd);
  return mf_launch_status();
}

// The rotation in neighbouring pairs (2i, 2i+1), in place: the first 2 `half` values of each of the
// first n_rot heads are rotated, whatever lies behind them in the head passes unchanged.
__global__ __launch_bounds__(256) void rope_pairs_inplace_kernel(float* __restrict__ x, const float* __restrict__ cs,
                                                                 const float* __restrict__ sn,
                                                                 const int* __restrict__ positions, int n_rot,
                                                                 int n_heads_total, int hd, int half) {
  const int t = blockIdx.x;
  const int pos = positions[t];
  float* row = x + (size_t)t * n_heads_total * hd;
  for (int it = threadIdx.x; it < n_rot * half; it += 256) {
    const int head = it / half, i = it % half;
    const float c = cs[(size_t)pos * half + i], s = sn[(size_t)pos * half + i];
    float* p = row + (size_t)head * hd + 2 * i;
    const float x0 = p[0], x1 = p[1];
    p[0] = x0 * c - x1 * s;
    p[1] = x1 * c + x0 * s;
  }
}

MF_API int mf_rope_pairs_inplace(float* x, const float* cs, const float* sn, const int* positions, int n_tok,
                                 int n_rot, int n_heads_total, int hd, int half, hipStream_t stream) {
  if (n_tok <= 0 || n_rot <= 0 || half <= 0) return 0;
  if (2 * half > hd || n_rot > n_heads_total || !cs || !sn) return (int)hipErrorInvalidValue;
  rope_pairs_inplace_kernel<<<n_tok, 256, 0, stream>>>(x, cs, sn, positions, n_rot, n_heads_total, hd, half);
  return mf_launch_status();
}

MF_API int mf_rope_kvwrite(const float* qkv, const float* cs, const float* sn, const int* positions,
                           const int* seq_of_tok, const int* page_table, int pt_stride, void* q_out,
                           void* kcache, void* vcache, int is_bf16, int n_tok, int nh, int nk, int hd,
                           int write_kv, hipStream_t stream) {
  if (n_tok <= 0) return 0;
  if ((cs == nullptr) != (sn == nullptr)) return (int)hipErrorInvalidValue;
  const bool vec = hd % 8 == 0 && (uintptr_t)qkv % 16 == 0 && (uintptr_t)cs % 16 == 0 && (uintptr_t)sn % 16 == 0 &&
                   (uintptr_t)q_out % 16 == 0 && (uintptr_t)kcache % 16 == 0 && (uintptr_t)vcache % 16 == 0;
  if (vec) {
    if (is_bf16)
      rope_kvwrite_vec_kernel<bf16, true><<<n_tok, 256, 0, stream>>>(qkv, cs, sn, positions, seq_of_tok, page_table,
                                                                     pt_stride, (bf16*)q_out, (bf16*)kcache,
                                                                     (bf16*)vcache, nh, nk, hd, write_kv);
    else
      rope_kvwrite_vec_kernel<float, false><<<n_tok, 256, 0, stream>>>(qkv, cs, sn, positions, seq_of_tok,
                                                                       page_table, pt_stride, (float*)q_out,
                                                                       (float*)kcache, (float*)vcache, nh, nk, hd,
                                                                       write_kv);
    return mf_launch_status();
  }
  dim3 grid(n_tok, write_kv ? nh + 2 * nk : nh);
  if (is_bf16)
    rope_kvwrite_kernel<bf16, true><<<grid, 64, 0, stream>>>(qkv, cs, sn, positions, seq_of_tok, page_table,
                                                       pt_stride, (bf16*)q_out, (bf16*)kcache,
                                                       (bf16*)vcache, nh, nk, hd, write_kv);
  else
    rope_kvwrite_kernel<float, false><<<grid, 64, 0, stream>>>(qkv, cs, sn, positions, seq_of_tok, page_table,
                                                        pt_stride, (float*)q_out, (float*)kcache,
                                                        (float*)vcache, nh, nk, hd, write_kv);
  return mf_launch_status();
}

// ---------------------------------------------------------------- seeded normal fill
// value(i) depends only on (seed, i) and is the same bits as the host's fill of the same
// (seed, i) (random_normal.h, host_random.cpp).  A thread makes both members of a pair.
template <typename OT>
__global__ __launch_bounds__(256) void fill_normal_kernel(OT* __restrict__ out, size_t n, uint64_t seed,
                                                          float std, int round_bf16) {
  const size_t pairs = (n + 1) / 2;
  for (size_t j = (size_t)blockIdx.x * 256 + threadIdx.x; j < pairs; j += (size_t)gridDim.x * 256) {
    double z0, z1;
    mf_normal_pair(seed, j, &z0, &z1);
    float v0, v1;
    {
#pragma clang fp contract(off)
      v0 = (float)z0 * std;
      v1 = (float)z1 * std;
    }
    if (round_bf16) {
      v0 = mf_bf16_value(mf_bf16_bits(v0));
      v1 = mf_bf16_value(mf_bf16_bits(v1));
    }
    out[2 * j] = from_f32<OT>(v0);
    if (2 * j + 1 < n) out[2 * j + 1] = from_f32<OT>(v1);
  }
}

// `round_bf16`: a float32 output holds values that bfloat16 represents (what a tensor written in
// bfloat16 and widened gives); a bfloat16 output is rounded in any case.
MF_API int mf_fill_normal(void* out, int is_bf16, size_t n, uint64_t seed, float std, int round_bf16,
                          hipStream_t stream) {
  if (n == 0) return 0;
  const size_t pairs = (n + 1) / 2;
  const int blocks = (int)((pairs + 255) / 256 < 16384 ? (pairs + 255) / 256 : 16384);
  if (is_bf16)
    fill_normal_kernel<bf16><<<blocks, 256, 0, stream>>>((bf16*)out, n, seed, std, 1);
  else
    fill_normal_kernel<float><<<blocks, 256, 0, stream>>>((float*)out, n, seed, std, round_bf16);
  return mf_launch_status();
}

// ---------------------------------------------------------------- table row + learned position row
// out[r][:] = table[ids[r]][:] + pos_table[positions[r]][:], added in 32-bit.  An id or a position
// outside its table gives a row of NaN, as `embed_kernel` does.
template <typename TT>
__global__ __launch_bounds__(256) void embed_pos_kernel(const TT* __restrict__ table, const TT* __restrict__ pos_table,
                                                        const int* __restrict__ ids, const int* __restrict__ positions,
                                                        float* __restrict__ out, int d, int vocab, int n_pos) {
  const int row = blockIdx.x;
  const int id = ids[row], p = positions[row];
  float* o = out + (size_t)row * d;
  if (id < 0 || id >= vocab || p < 0 || p >= n_pos) {
    for (int i = threadIdx.x; i < d; i += 256) o[i] = __builtin_nanf("");
    return;
  }
  const TT* src = table + (size_t)id * d;
  const TT* ps = pos_table + (size_t)p * d;
  for (int i = threadIdx.x; i < d; i += 256) o[i] = to_f32(src[i]) + to_f32(ps[i]);
}

MF_API int mf_embed_pos(const void* table, const void* pos_table, int tables_are_bf16, const int* ids,
                        const int* positions, float* out, int rows, int d, int vocab, int n_pos, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (tables_are_bf16)
    embed_pos_kernel<bf16><<<rows, 256, 0, stream>>>((const bf16*)table, (const bf16*)pos_table, ids, positions, out, d,
                                                      vocab, n_pos);
  else
    embed_pos_kernel<float><<<rows, 256, 0, stream>>>((const float*)table, (const float*)pos_table, ids, positions, out,
                                                       d, vocab, n_pos);
  return mf_launch_status();
}

// ---------------------------------------------------------------- gelu, tanh form
// 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3))), from 32-bit sums, rounded once.
__device__ __forceinline__ float gelu_tanh_of(float z) {
  return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}
template <typename OT>
__global__ __launch_bounds__(256) void gelu_tanh_kernel(const float* __restrict__ x, OT* __restrict__ out, size_t n) {
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i < n) out[i] = from_f32<OT>(gelu_tanh_of(x[i]));
}

MF_API int mf_gelu_tanh(const float* x, void* out, int out_is_bf16, size_t n, hipStream_t stream) {
  if (n == 0) return 0;
  const unsigned blocks = (unsigned)((n + 255) / 256);
  if (out_is_bf16)
    gelu_tanh_kernel<bf16><<<blocks, 256, 0, stream>>>(x, (bf16*)out, n);
  else
    gelu_tanh_kernel<float><<<blocks, 256, 0, stream>>>(x, (float*)out, n);
  return mf_launch_status();
}

// ---------------------------------------------------------------- capped logits
// x <- cap tanh(x / cap), in place, 32-bit.
__global__ __launch_bounds__(256) void softcap_kernel(float* __restrict__ x, float cap, float inv_cap, size_t n) {
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i < n) x[i] = cap * tanhf(x[i] * inv_cap);
}

MF_API int mf_softcap(float* x, float cap, size_t n, hipStream_t stream) {
  if (n == 0) return 0;
  if (!(cap > 0.f)) return (int)hipErrorInvalidValue;
  softcap_kernel<<<(unsigned)((n + 255) / 256), 256, 0, stream>>>(x, cap, 1.0f / cap, n);
  return mf_launch_status();
}

// ---------------------------------------------------------------- weighted sum of row buffers
// out[r][:] = sum_j w[j] x_j[row(j, r)][:], added in the order of j.  The first `n_indexed` buffers are
// read at row row_idx[r] (they hold more rows than `out`), the others at row r.  Up to MF_WSUM_MAX
// buffers a launch; the entry point chains launches for more (the later ones add onto `out`).
#define MF_WSUM_MAX 32
struct WsumPtrs { const float* p[MF_WSUM_MAX]; };
__global__ __launch_bounds__(256) void weighted_sum_kernel(WsumPtrs src, int n, int n_indexed,
                                                           const int* __restrict__ row_idx, const float* __restrict__ w,
                                                           float* __restrict__ out, int d, int add) {
  const int r = blockIdx.x;
  const int ri = row_idx ? row_idx[r] : r;
  float* o = out + (size_t)r * d;
  const int i = blockIdx.y * 256 + threadIdx.x;
  if (i >= d) return;
  float v[MF_WSUM_MAX];
#pragma unroll
  for (int j = 0; j < MF_WSUM_MAX; ++j)          // all loads first: one trip to memory
    v[j] = j < n ? src.p[j][(size_t)(j < n_indexed ? ri : r) * d + i] : 0.f;
  float a = add ? o[i] : 0.f;
#pragma unroll
  for (int j = 0; j < MF_WSUM_MAX; ++j)
    if (j < n) a = fmaf(w[j], v[j], a);
  o[i] = a;
}

// `ptrs`: host array of n device pointers
MF_API int mf_weighted_sum(const void* const* ptrs, int n, int n_indexed, const int* row_idx, const float* w, float* out,
                           int rows, int d, hipStream_t stream) {
  if (rows <= 0 || d <= 0) return 0;
  if (n <= 0 || !ptrs || !w || !out) return (int)hipErrorInvalidValue;
  for (int j0 = 0; j0 < n; j0 += MF_WSUM_MAX) {
    WsumPtrs a;
    const int m = n - j0 < MF_WSUM_MAX ? n - j0 : MF_WSUM_MAX;
    for (int j = 0; j < MF_WSUM_MAX; ++j) a.p[j] = j < m ? (const float*)ptrs[j0 + j] : nullptr;
    const int idx = n_indexed - j0 < 0 ? 0 : (n_indexed - j0 > m ? m : n_indexed - j0);
    weighted_sum_kernel<<<dim3(rows, (d + 255) / 256), 256, 0, stream>>>(a, m, idx, row_idx, w + j0, out, d, j0 > 0 ? 1 : 0);
    const int rc = mf_launch_status();
    if (rc) return rc;
  }
  return 0;
}

// ---------------------------------------------------------------- rows added into rows
// h[r][:] += x[r][:], both 32-bit (an earlier state of the residual stream that joins it again)
__global__ __launch_bounds__(256) void add_rows_kernel(float* __restrict__ h, const float* __restrict__ x, size_t n) {
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i < n) h[i] += x[i];
}

MF_API int mf_add_rows(float* h, const float* x, size_t n, hipStream_t stream) {
  if (n == 0) return 0;
  add_rows_kernel<<<(unsigned)((n + 255) / 256), 256, 0, stream>>>(h, x, n);
  return mf_launch_status();
}

// ---------------------------------------------------------------- square of relu
template <typename OT>
__global__ __launch_bounds__(256) void relu2_kernel(const float* __restrict__ x, OT* __restrict__ out, size_t n) {
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i < n) {
    const float z = fmaxf(x[i], 0.f);
    out[i] = from_f32<OT>(z * z);
  }
}
// the same, four values a thread
template <typename OT>
__global__ __launch_bounds__(256) void relu2_vec_kernel(const float* __restrict__ x, OT* __restrict__ out, size_t n4) {
  typedef OT out4 __attribute__((ext_vector_type(4)));
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i < n4) {
    const float4 v = ((const float4*)x)[i];
    const float a = fmaxf(v.x, 0.f), b = fmaxf(v.y, 0.f), c = fmaxf(v.z, 0.f), d = fmaxf(v.w, 0.f);
    ((out4*)out)[i] = out4{from_f32<OT>(a * a), from_f32<OT>(b * b), from_f32<OT>(c * c), from_f32<OT>(d * d)};
  }
}

MF_API int mf_relu2(const float* x, void* out, int out_is_bf16, size_t n, hipStream_t stream) {
  if (n == 0) return 0;
  if (n % 4 == 0) {
    const unsigned blocks = (unsigned)((n / 4 + 255) / 256);
    if (out_is_bf16)
      relu2_vec_kernel<bf16><<<blocks, 256, 0, stream>>>(x, (bf16*)out, n / 4);
    else
      relu2_vec_kernel<float><<<blocks, 256, 0, stream>>>(x, (float*)out, n / 4);
    return mf_launch_status();
  }
  const unsigned blocks = (unsigned)((n + 255) / 256);
  if (out_is_bf16)
    relu2_kernel<bf16><<<blocks, 256, 0, stream>>>(x, (bf16*)out, n);
  else
    relu2_kernel<float><<<blocks, 256, 0, stream>>>(x, (float*)out, n);
  return mf_launch_status();
}

// ---------------------------------------------------------------- layer norm, alone or behind a scaled sum
// u = x[row] (JOIN: alpha x[row] + y[row]); out = (u - mean(u)) / sqrt(mean((u - mean(u))^2) + eps) * w.  JOIN
// writes the 32-bit stream, which may be x itself, and with `cast_out` its rounded copy.  A row of at most
// 256 * 4 * KEEP values, a multiple of 4 of them, stays in registers; other rows are read once per pass (each
// thread reads and writes its own values only, so in place is fine).
template <typename OT, bool JOIN, int KEEP>
__global__ __launch_bounds__(256) void layernorm_kernel(const float* x, const float* __restrict__ y, float alpha,
                                                        const int* __restrict__ row_idx, const float* __restrict__ w,
                                                        OT* out, bf16* __restrict__ cast_out, int d, float eps) {
  __shared__ float scratch[4];
  const int row = blockIdx.x;
  const float* xr = x + (size_t)(row_idx ? row_idx[row] : row) * d;
  const float* yr = JOIN ? y + (size_t)row * d : nullptr;
  OT* o = out + (size_t)row * d;
  bf16* co = cast_out ? cast_out + (size_t)row * d : nullptr;
  if (KEEP > 0) {
    typedef OT out4 __attribute__((ext_vector_type(4)));
    float4 v[KEEP > 0 ? KEEP : 1];
    float s = 0.f;
#pragma unroll
    for (int c = 0; c < KEEP; ++c) {
      const int i = (c * 256 + threadIdx.x) * 4;
      v[c] = make_float4(0.f, 0.f, 0.f, 0.f);
      if (i < d) {
        v[c] = *reinterpret_cast<const float4*>(xr + i);
        if (JOIN) {
          const float4 b = *reinterpret_cast<const float4*>(yr + i);
          v[c].x = fmaf(alpha, v[c].x, b.x);
          v[c].y = fmaf(alpha, v[c].y, b.y);
          v[c].z = fmaf(alpha, v[c].z, b.z);
          v[c].w = fmaf(alpha, v[c].w, b.w);
        }
      }
      s += (v[c].x + v[c].y) + (v[c].z + v[c].w);
    }
    const float mean = block_sum<256>(s, scratch) / (float)d;
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < KEEP; ++c) {
      if ((c * 256 + (int)threadIdx.x) * 4 < d) {
        v[c].x -= mean;
        v[c].y -= mean;
        v[c].z -= mean;
        v[c].w -= mean;
      }
      ss = fmaf(v[c].x, v[c].x, ss);
      ss = fmaf(v[c].y, v[c].y, ss);
      ss = fmaf(v[c].z, v[c].z, ss);
      ss = fmaf(v[c].w, v[c].w, ss);
    }
    const float r = 1.0f / sqrtf(block_sum<256>(ss, scratch) / (float)d + eps);
#pragma unroll
    for (int c = 0; c < KEEP; ++c) {
      const int i = (c * 256 + threadIdx.x) * 4;
      if (i < d) {
        const float4 g = *reinterpret_cast<const float4*>(w + i);
        const float4 z = make_float4(v[c].x * r * g.x, v[c].y * r * g.y, v[c].z * r * g.z, v[c].w * r * g.w);
        *reinterpret_cast<out4*>(o + i) = out4{from_f32<OT>(z.x), from_f32<OT>(z.y), from_f32<OT>(z.z), from_f32<OT>(z.w)};
        if (co) *reinterpret_cast<bf16x4*>(co + i) = bf16x4{(bf16)z.x, (bf16)z.y, (bf16)z.z, (bf16)z.w};
      }
    }
    return;
  }
  auto value = [&](int i) { return JOIN ? fmaf(alpha, xr[i], yr[i]) : xr[i]; };
  float s = 0.f;
  for (int i = threadIdx.x; i < d; i += 256) s += value(i);
  const float mean = block_sum<256>(s, scratch) / (float)d;
  float ss = 0.f;
  for (int i = threadIdx.x; i < d; i += 256) {
    const float c = value(i) - mean;
    ss = fmaf(c, c, ss);
  }
  const float r = 1.0f / sqrtf(block_sum<256>(ss, scratch) / (float)d + eps);
  for (int i = threadIdx.x; i < d; i += 256) {
    const float z = (value(i) - mean) * r * w[i];
    o[i] = from_f32<OT>(z);
    if (co) co[i] = (bf16)z;
  }
}

template <typename OT, bool JOIN>
static int launch_layernorm(const float* x, const float* y, float alpha, const int* row_idx, const float* w, OT* out,
                            bf16* cast_out, int rows, int d, float eps, hipStream_t stream) {
#define MF_GO(KEEP) \
  layernorm_kernel<OT, JOIN, KEEP><<<rows, 256, 0, stream>>>(x, y, alpha, row_idx, w, out, cast_out, d, eps)
  if (d % 4 != 0 || d > 8192) MF_GO(0);
  else if (d <= 1024) MF_GO(1);
  else if (d <= 2048) MF_GO(2);
  else if (d <= 4096) MF_GO(4);
  else MF_GO(8);
#undef MF_GO
  return mf_launch_status();
}

MF_API int mf_layernorm(const float* x, const int* row_idx, const float* w, void* out, int out_is_bf16, int rows, int d,
                        float eps, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (d <= 0) return (int)hipErrorInvalidValue;
  if (out_is_bf16)
    return launch_layernorm<bf16, false>(x, nullptr, 1.f, row_idx, w, (bf16*)out, nullptr, rows, d, eps, stream);
  return launch_layernorm<float, false>(x, nullptr, 1.f, row_idx, w, (float*)out, nullptr, rows, d, eps, stream);
}

// h <- layernorm(alpha h + y) in place; cast_out (bfloat16, or null) gets the new rows rounded
MF_API int mf_layernorm_join(float* h, const float* y, float alpha, const float* w, void* cast_out, int rows, int d, float eps,
                             hipStream_t stream) {
  if (rows <= 0) return 0;
  if (d <= 0) return (int)hipErrorInvalidValue;
  return launch_layernorm<float, true>(h, y, alpha, nullptr, w, h, (bf16*)cast_out, rows, d, eps, stream);
}

// ---------------------------------------------------------------- two normed rows, summed
// out[r] (+)= scale (a[r] / rms(a[r]) wa + b[r] / rms(b[r]) wb), rms with eps inside the root
template <int KEEP>
__global__ __launch_bounds__(256) void rmsnorm_pair_kernel(const float* __restrict__ a, const float* __restrict__ wa,
                                                           const float* __restrict__ b, const float* __restrict__ wb,
                                                           float* __restrict__ out, int d, float eps, float scale, int add) {
  __shared__ float scratch[4];
  const size_t at = (size_t)blockIdx.x * d;
  float va[KEEP > 0 ? KEEP : 1], vb[KEEP > 0 ? KEEP : 1];
  float sa = 0.f, sb = 0.f;
  if (KEEP > 0) {
#pragma unroll
    for (int c = 0; c < KEEP; ++c) {
      const int i = c * 256 + threadIdx.x;
      va[c] = i < d ? a[at + i] : 0.f;
      vb[c] = i < d ? b[at + i] : 0.f;
      sa = fmaf(va[c], va[c], sa);
      sb = fmaf(vb[c], vb[c], sb);
    }
  } else {
    for (int i = threadIdx.x; i < d; i += 256) {
      sa = fmaf(a[at + i], a[at + i], sa);
      sb = fmaf(b[at + i], b[at + i], sb);
    }
  }
  const float ra = scale / sqrtf(block_sum<256>(sa, scratch) / (float)d + eps);
  const float rb = scale / sqrtf(block_sum<256>(sb, scratch) / (float)d + eps);
  auto put = [&](int i, float x, float z) {
    const float v = x * ra * wa[i] + z * rb * wb[i];
    out[at + i] = add ? out[at + i] + v : v;
  };
  if (KEEP > 0) {
#pragma unroll
    for (int c = 0; c < KEEP; ++c) {
      const int i = c * 256 + threadIdx.x;
      if (i < d) put(i, va[c], vb[c]);
    }
  } else {
    for (int i = threadIdx.x; i < d; i += 256) put(i, a[at + i], b[at + i]);
  }
}

MF_API int mf_rmsnorm_pair(const float* a, const float* wa, const float* b, const float* wb, float* out, int rows, int d,
                           float eps, float scale, int add, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (d <= 0) return (int)hipErrorInvalidValue;
  if (d <= 2048)
    rmsnorm_pair_kernel<8><<<rows, 256, 0, stream>>>(a, wa, b, wb, out, d, eps, scale, add);
  else if (d <= 4096)
    rmsnorm_pair_kernel<16><<<rows, 256, 0, stream>>>(a, wa, b, wb, out, d, eps, scale, add);
  else
    rmsnorm_pair_kernel<0><<<rows, 256, 0, stream>>>(a, wa, b, wb, out, d, eps, scale, add);
  return mf_launch_status();
}
