// Kernels of the model families with several residual streams per token, differential attention heads and the generalised
// delta rule (all fp32, both serving dtypes; step metadata cu_q / kv_lens / slot_ids as in seqmix.hip):
//
//   mi_stream_mix        one launch per sublayer boundary: the last sublayer's output mixed into the streams, the next
//                        sublayer's input read from them, RMS-normed in groups of channels, shifted towards the previous
//                        token's (carried per sequence slot)
//   mi_diff_heads        a1 - lambda a2 of a head's two attention maps, its unit norm, a gate number per head
//   mi_general_delta     S <- diag(w) S - (a u) (u^T S) + k v^T,  o = S^T r, the state in per-sequence slots
#include "seqmix_common.hpp"

namespace mi {

// ---------------------------------------------------------------------------------------------------------------
// residual streams
// ---------------------------------------------------------------------------------------------------------------
template <int VEC>
struct FVec;
template <>
struct FVec<1> {
  float v[1];
};
template <>
struct __attribute__((aligned(16))) FVec<4> {
  float v[4];
};
template <int VEC>
__device__ __forceinline__ FVec<VEC> ldv(const float* p) { return *reinterpret_cast<const FVec<VEC>*>(p); }
template <int VEC>
__device__ __forceinline__ void stv(float* p, const FVec<VEC>& x) { *reinterpret_cast<FVec<VEC>*>(p) = x; }

struct StreamMixArgs {
  const float* src;
  int64_t ld_src, src_stride;
  float* dst;
  int64_t ld_dst, dst_stride;
  const float* y;
  int64_t ldy;
  const float* mix;       // [NS][NS], from x to
  const float* out_coef;  // [NS]
  const float* in_coef;   // [NS] or nullptr: ones
  const float* norm_w;
  int groups;
  float eps;
  const float* shift;
  float* shift_state;  // [slots][width]
  float* carry;        // [n_seqs][width]; nullptr: one row per sequence, the state is advanced here
  const int32_t* cu_q;
  const int32_t* kv_lens;
  const int32_t* slot_ids;
  int n_seqs;
  float* h;
  int64_t ldh;
  int rows, width, rows_per_group;
};

// A workgroup takes rows_per_group consecutive rows, one after the other.  With the shift, a row needs the h of the row
// before it: it is still in LDS from the row before; for the workgroup's first row (unless that starts its sequence's
// step) it is computed again from that row's old streams - which is why the new streams go to another buffer then.  What
// the sequence's last row leaves for the next step goes through `carry`: the slot's state is still being read.
template <int NS, int VEC>
__global__ __launch_bounds__(256) void stream_mix_kernel(StreamMixArgs a) {
  extern __shared__ __attribute__((aligned(16))) float smem[];  // h of this row and of the row before; partial sums
  const int W = a.width, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const bool shifted = a.shift != nullptr;
  float* red = smem + (shifted ? 2 : 1) * (int64_t)W;
  float inc[NS], outc[NS], mx[NS][NS];
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    inc[i] = a.in_coef ? a.in_coef[i] : 1.f;
    outc[i] = a.y ? a.out_coef[i] : 0.f;
#pragma unroll
    for (int j = 0; j < NS; ++j) mx[i][j] = a.y ? a.mix[i * NS + j] : 0.f;
  }
  const int part = W / a.groups;
  const int wpg = a.groups == 1 ? 4 : a.groups == 2 ? 2 : 1;  // waves that share a group's sum
  const int r0 = blockIdx.x * a.rows_per_group, r1 = min(r0 + a.rows_per_group, a.rows);
  int s = 0, first = r0;
  if (shifted) {
    s = seq_of_row(a.cu_q, a.n_seqs, r0);
    if (r0 > a.cu_q[s]) first = r0 - 1;
  }
  float* cur = smem;
  float* prev = shifted ? smem + W : smem;
  for (int row = first; row < r1; ++row) {
    const bool mine = row >= r0;
    if (shifted)
      while (s + 1 < a.n_seqs && row >= a.cu_q[s + 1]) ++s;
    const float* xs = a.src + (int64_t)row * a.ld_src;
    float* xd = a.dst && mine ? a.dst + (int64_t)row * a.ld_dst : nullptr;
    const float* yr = a.y ? a.y + (int64_t)row * a.ldy : nullptr;
    for (int c = tid * VEC; c < W; c += 256 * VEC) {
      FVec<VEC> x[NS], u;
#pragma unroll
      for (int i = 0; i < NS; ++i) x[i] = ldv<VEC>(xs + (int64_t)i * a.src_stride + c);
      if (yr) {
        const FVec<VEC> yv = ldv<VEC>(yr + c);
        FVec<VEC> z[NS];
#pragma unroll
        for (int j = 0; j < NS; ++j)
#pragma unroll
          for (int e = 0; e < VEC; ++e) {
            float t = mx[0][j] * x[0].v[e];
#pragma unroll
            for (int i = 1; i < NS; ++i) t = fmaf(mx[i][j], x[i].v[e], t);
            z[j].v[e] = fmaf(outc[j], yv.v[e], t);
          }
#pragma unroll
        for (int j = 0; j < NS; ++j) x[j] = z[j];
      }
      if (xd) {
#pragma unroll
        for (int j = 0; j < NS; ++j) stv<VEC>(xd + (int64_t)j * a.dst_stride + c, x[j]);
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        float t = inc[0] * x[0].v[e];
#pragma unroll
        for (int i = 1; i < NS; ++i) t = fmaf(inc[i], x[i].v[e], t);
        u.v[e] = t;
      }
      stv<VEC>(cur + c, u);
    }
    if (a.norm_w) {
      __syncthreads();
      for (int un = wave; un < a.groups * wpg; un += 4) {
        const float* p = cur + (un / wpg) * part;
        float sq = 0.f;
        for (int i = (un % wpg) * 64 + lane; i < part; i += 64 * wpg) sq = fmaf(p[i], p[i], sq);
        sq = wave_sum(sq);
        if (lane == 0) red[un] = sq;
      }
      __syncthreads();
    }
    const bool starts = shifted && row == a.cu_q[s], ends = shifted && row + 1 == a.cu_q[s + 1];
    const bool from_state = starts && a.kv_lens[s] - (a.cu_q[s + 1] - a.cu_q[s]) > 0;
    float* st = shifted ? a.shift_state + (int64_t)a.slot_ids[s] * W : nullptr;
    float* hr = a.h + (int64_t)row * a.ldh;
    int g_have = -1;
    float rstd = 1.f;
    for (int c = tid * VEC; c < W; c += 256 * VEC) {
      FVec<VEC> u = ldv<VEC>(cur + c);
      if (a.norm_w) {
        const int g = c / part;
        if (g != g_have) {
          float sq = 0.f;
          for (int i = 0; i < wpg; ++i) sq += red[g * wpg + i];
          rstd = 1.f / sqrtf(sq / (float)part + a.eps);
          g_have = g;
        }
        const FVec<VEC> w = ldv<VEC>(a.norm_w + c);
#pragma unroll
        for (int e = 0; e < VEC; ++e) u.v[e] = u.v[e] * rstd * w.v[e];
      }
      if (shifted) {
        FVec<VEC> p = {};
        if (!starts) p = ldv<VEC>(prev + c);
        else if (from_state) p = ldv<VEC>(st + c);
        stv<VEC>(cur + c, u);
        if (ends && mine) stv<VEC>(a.carry ? a.carry + (int64_t)s * W + c : st + c, u);
        const FVec<VEC> sh = ldv<VEC>(a.shift + c);
#pragma unroll
        for (int e = 0; e < VEC; ++e) u.v[e] = fmaf(p.v[e] - u.v[e], sh.v[e], u.v[e]);
      }
      if (mine) stv<VEC>(hr + c, u);
    }
    if (shifted) {
      float* t = cur;
      cur = prev;
      prev = t;
    } else if (a.norm_w) {
      __syncthreads();  // (the one buffer is written again; a thread's own elements are all it reads without a norm)
    }
  }
}

__global__ __launch_bounds__(256) void stream_carry_kernel(const float* __restrict__ carry, float* __restrict__ state,
                                                           const int32_t* __restrict__ cu_q,
                                                           const int32_t* __restrict__ slot_ids, int width) {
  const int s = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
  if (c >= width || cu_q[s + 1] == cu_q[s]) return;
  state[(int64_t)slot_ids[s] * width + c] = carry[(int64_t)s * width + c];
}

// ---------------------------------------------------------------------------------------------------------------
// differential heads: a workgroup per row, a wave per head in turn; lambda once per wave
// ---------------------------------------------------------------------------------------------------------------
template <int VPL>  // value channels per lane
__global__ __launch_bounds__(256) void diff_heads_kernel(const float* __restrict__ o, int64_t ldo_in,
                                                         const float* __restrict__ lam, int D, float diff, float eps,
                                                         const float* __restrict__ gate, int64_t ldg,
                                                         float* __restrict__ out, int64_t ldo, int H, int G, int Dv) {
  const int64_t row = blockIdx.x;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int rep = H / G;
  float d1 = 0.f, d2 = 0.f;
  for (int i = lane; i < D; i += 64) {
    d1 = fmaf(lam[i], lam[D + i], d1);
    d2 = fmaf(lam[2 * D + i], lam[3 * D + i], d2);
  }
  const float l = expf(wave_sum(d1)) - expf(wave_sum(d2)) + diff;
  for (int h = wave; h < H; h += 4) {
    const float* a1 = o + row * ldo_in + (int64_t)((h / rep) * 2 * rep + h % rep) * Dv;
    const float* a2 = a1 + (int64_t)rep * Dv;
    float v[VPL], sq = 0.f;
#pragma unroll
    for (int i = 0; i < VPL; ++i) {
      const int d = lane + 64 * i;
      v[i] = d < Dv ? fmaf(-l, a2[d], a1[d]) : 0.f;
      sq = fmaf(v[i], v[i], sq);
    }
    float mult = (1.f - diff) / sqrtf(wave_sum(sq) / (float)Dv + eps);
    if (gate) mult *= sigmoid_f(gate[row * ldg + h]);
    float* dst = out + row * ldo + (int64_t)h * Dv;
#pragma unroll
    for (int i = 0; i < VPL; ++i) {
      const int d = lane + 64 * i;
      if (d < Dv) dst[d] = v[i] * mult;
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------
// generalised delta rule
// ---------------------------------------------------------------------------------------------------------------
// k = |k| u, so the rule per value column is  S_i <- w_i S_i + u_i (|k| v - a_i dot),  dot = sum_i u_i S_i over the old
// column.  The dot for row t + 1 is summed while row t's new column is formed: ONE pass over the state per row, with two
// independent sums (read-out and next dot) whose cross-lane ends overlap - a two-pass walk waits for the dot before it may
// touch the state.
// A workgroup = 32 value columns of one (sequence, head); LANES lanes share CPL columns, lane r keeping the key channels
// (LANES jj + r) * 4 + e of them in registers for the whole walk over the step's rows.  ROWS rows at a time go through LDS,
// fetched one batch ahead and turned into r, u, w, a and |k| v on the way: the staging lanes of a row sum its k^2 among
// themselves.  A full batch is walked by unrolled code, so that the LDS reads of later rows run ahead of the walk.  (8
// sequences x 1024 rows x 8 heads x 128 channels, 16 lanes: one column per lane group 285 us, two 435 us, 8 lanes 350 us; not
// unrolled 430 us.)  State in thread order, 16-byte pieces.
constexpr int kGdCols = 32;

template <int LANES>
__device__ __forceinline__ float lanes_sum(float v) {  // over the LANES neighbours that share a column
  v = xor_sum<4>(xor_sum<2>(xor_sum<1>(v)));
  if constexpr (LANES == 16) v = xor_sum<8>(v);
  return v;
}

template <int LANES, int DR, int CPL, int ROWS>  // DR: key channels per lane
__global__ __launch_bounds__(LANES* kGdCols / CPL) void general_delta_kernel(
    const float* __restrict__ proj, int64_t ld, int r_off, int k_off, int v_off, int a_off, const float* __restrict__ wdec,
    int64_t ldw, float* __restrict__ state, const int32_t* __restrict__ cu_q, const int32_t* __restrict__ kv_lens,
    const int32_t* __restrict__ slot_ids, int H, int D, int Dv, float* __restrict__ out, int64_t ldo) {
  constexpr int NT = LANES * kGdCols / CPL, DP = LANES * DR, SL = NT / ROWS, PE = DP / SL, JJ = DR / 4;
  static_assert(SL * ROWS == NT && (SL == 8 || SL == 16 || SL == 32) && DP % SL == 0 && kGdCols % SL == 0, "staging shape");
  __shared__ __attribute__((aligned(16))) float rs[ROWS][DP];
  __shared__ __attribute__((aligned(16))) float us[ROWS][DP];
  __shared__ __attribute__((aligned(16))) float ws[ROWS][DP];
  __shared__ __attribute__((aligned(16))) float as[ROWS][DP];
  __shared__ float vs[ROWS][kGdCols];
  const int s = blockIdx.x, h = blockIdx.y, cb = blockIdx.z;
  const int tid = threadIdx.x, r = tid & (LANES - 1), cg = tid / LANES;
  const int r0 = cu_q[s], n = cu_q[s + 1] - r0;
  if (n == 0) return;
  const int start = kv_lens[s] - n;
  float* slot = state + (((int64_t)slot_ids[s] * H + h) * gridDim.z + cb) * (int64_t)(DP * kGdCols);
  float st[CPL][DR];
#pragma unroll
  for (int cc = 0; cc < CPL; ++cc)
#pragma unroll
    for (int jj = 0; jj < JJ; ++jj) {
      float4 x{0.f, 0.f, 0.f, 0.f};
      if (start > 0) x = *reinterpret_cast<const float4*>(slot + ((cc * JJ + jj) * NT + tid) * 4);
      st[cc][jj * 4 + 0] = x.x, st[cc][jj * 4 + 1] = x.y, st[cc][jj * 4 + 2] = x.z, st[cc][jj * 4 + 3] = x.w;
    }
  const int pt = tid / SL, ps = tid % SL;
  float fr[PE], fk[PE], fa[PE], fw[PE], fv[kGdCols / SL];
  auto fetch = [&](int c0) {
    const bool live = c0 + pt < n;
    const int64_t row = r0 + (live ? c0 + pt : 0);
    const float* p = proj + row * ld;
    const float* wp = wdec + row * ldw + h * D;
#pragma unroll
    for (int m = 0; m < PE; ++m) {
      const int i = ps + SL * m;
      const bool ok = live && i < D;
      fr[m] = ok ? p[r_off + h * D + i] : 0.f;
      fk[m] = ok ? p[k_off + h * D + i] : 0.f;
      fa[m] = ok ? p[a_off + h * D + i] : 0.f;
      fw[m] = ok ? wp[i] : 0.f;
    }
#pragma unroll
    for (int m = 0; m < kGdCols / SL; ++m) {
      const int c = cb * kGdCols + ps + SL * m;
      fv[m] = live && c < Dv ? p[v_off + h * Dv + c] : 0.f;
    }
  };
  fetch(0);
  for (int c0 = 0; c0 < n; c0 += ROWS) {
    float sq = 0.f;
#pragma unroll
    for (int m = 0; m < PE; ++m) sq = fmaf(fk[m], fk[m], sq);
    sq = lanes_sum<(SL >= 16 ? 16 : 8)>(sq);
    if constexpr (SL == 32) sq = xor_sum<16>(sq);
    const float len = sqrtf(sq + 1e-6f), inv = 1.f / len;
    __syncthreads();  // the previous rows' vectors have been consumed
#pragma unroll
    for (int m = 0; m < PE; ++m) {
      const int i = ps + SL * m;
      rs[pt][i] = fr[m], us[pt][i] = fk[m] * inv, ws[pt][i] = fw[m], as[pt][i] = fa[m];
    }
#pragma unroll
    for (int m = 0; m < kGdCols / SL; ++m) vs[pt][ps + SL * m] = fv[m] * len;
    __syncthreads();
    if (c0 + ROWS < n) fetch(c0 + ROWS);
    const int nt = min(ROWS, n - c0);
    auto load = [&](const float(&m)[ROWS][DP], int t, float(&x)[DR]) {
#pragma unroll
      for (int jj = 0; jj < JJ; ++jj) {
        const float4 q = reinterpret_cast<const float4*>(m[t])[jj * LANES + r];
        x[jj * 4 + 0] = q.x, x[jj * 4 + 1] = q.y, x[jj * 4 + 2] = q.z, x[jj * 4 + 3] = q.w;
      }
    };
    float u[DR], dot[CPL];
    load(us, 0, u);
#pragma unroll
    for (int cc = 0; cc < CPL; ++cc) {  // the batch's first dot: a pass of its own
      float d0 = 0.f, d1 = 0.f;
#pragma unroll
      for (int e = 0; e < DR; e += 2) d0 = fmaf(u[e], st[cc][e], d0), d1 = fmaf(u[e + 1], st[cc][e + 1], d1);
      dot[cc] = lanes_sum<LANES>(d0 + d1);
    }
    auto step = [&](int t, int t_next) {
      float un[DR], rr[DR], ww[DR], aa[DR];
      load(us, t_next, un), load(rs, t, rr), load(ws, t, ww), load(as, t, aa);
      float o0[CPL], o1[CPL], d0[CPL], d1[CPL];
#pragma unroll
      for (int cc = 0; cc < CPL; ++cc) {
        const float v = vs[t][cg * CPL + cc];
        o0[cc] = o1[cc] = d0[cc] = d1[cc] = 0.f;
#pragma unroll
        for (int e = 0; e < DR; ++e) {
          float& S = st[cc][e];
          S = fmaf(ww[e], S, u[e] * fmaf(-aa[e], dot[cc], v));
          float& o = e & 1 ? o1[cc] : o0[cc];
          float& d = e & 1 ? d1[cc] : d0[cc];
          o = fmaf(rr[e], S, o);
          d = fmaf(un[e], S, d);
        }
      }
#pragma unroll
      for (int cc = 0; cc < CPL; ++cc) dot[cc] = lanes_sum<LANES>(d0[cc] + d1[cc]);
#pragma unroll
      for (int cc = 0; cc < CPL; ++cc) {
        const float o = lanes_sum<LANES>(o0[cc] + o1[cc]);
        const int c = cb * kGdCols + cg * CPL + cc;
        if (r == 0 && c < Dv) out[(int64_t)(r0 + c0 + t) * ldo + h * Dv + c] = o;
      }
#pragma unroll
      for (int e = 0; e < DR; ++e) u[e] = un[e];
    };
    if (nt == ROWS) {  // unrolled: the rows' LDS reads run ahead of the walk
#pragma unroll
      for (int t = 0; t < ROWS; ++t) step(t, t + 1 < ROWS ? t + 1 : t);
    } else {
      for (int t = 0; t < nt; ++t) step(t, min(t + 1, nt - 1));
    }
  }
#pragma unroll
  for (int cc = 0; cc < CPL; ++cc)
#pragma unroll
    for (int jj = 0; jj < JJ; ++jj)
      *reinterpret_cast<float4*>(slot + ((cc * JJ + jj) * NT + tid) * 4) =
          float4{st[cc][jj * 4 + 0], st[cc][jj * 4 + 1], st[cc][jj * 4 + 2], st[cc][jj * 4 + 3]};
}

template <int NS>
static void launch_stream(const StreamMixArgs& a, bool vec, int groups, size_t lds, hipStream_t st) {
  if (vec) hipLaunchKernelGGL((stream_mix_kernel<NS, 4>), dim3(groups), dim3(256), lds, st, a);
  else hipLaunchKernelGGL((stream_mix_kernel<NS, 1>), dim3(groups), dim3(256), lds, st, a);
}

}  // namespace mi

using namespace mi;

extern "C" int mi_stream_mix(const float* src, int64_t ld_src, int64_t src_stride, float* dst, int64_t ld_dst,
                             int64_t dst_stride, int n_streams, const float* y, int64_t ldy, const float* mix,
                             const float* out_coef, const float* in_coef, const float* norm_w, int groups, float eps,
                             const float* shift, float* shift_state, float* carry, const int32_t* cu_q,
                             const int32_t* kv_lens, const int32_t* slot_ids, int n_seqs, int max_rows_per_seq, float* h,
                             int64_t ldh, int rows, int width, mi_stream stream) {
  if (!src || !h || rows < 0 || width < 1 || n_streams < 1 || groups < 1 || width % groups) return MI_EINVAL;
  if (src_stride != 0 && src_stride < width) return MI_EINVAL;
  if (ld_src < src_stride * (n_streams - 1) + width || ldh < width) return MI_EINVAL;
  if (dst && (dst_stride < width || ld_dst < dst_stride * (n_streams - 1) + width)) return MI_EINVAL;
  if (y && (ldy < width || !mix || !out_coef)) return MI_EINVAL;
  if (dst == src && dst && (ld_dst != ld_src || dst_stride != src_stride)) return MI_EINVAL;
  const bool several = shift && max_rows_per_seq > 1;
  if (shift && (!shift_state || !cu_q || !kv_lens || !slot_ids || n_seqs < 1 || max_rows_per_seq < 1)) return MI_EINVAL;
  if (several && (!carry || dst == src)) return MI_EINVAL;
  if (n_streams > 8 || width > 8000 || n_seqs > 65535) return MI_EUNSUPPORTED;
  if (rows == 0) return MI_OK;
  const int per = several ? (rows < 2048 ? 1 : rows >= 8192 ? 8 : rows / 1024) : 1;
  StreamMixArgs a{src, ld_src, src_stride, dst, ld_dst, dst_stride, y, ldy, mix, out_coef, in_coef, norm_w, groups, eps, shift,
                  shift_state, several ? carry : nullptr, cu_q, kv_lens, slot_ids, n_seqs, h, ldh, rows, width, per};
  bool vec = width % 4 == 0 && (width / groups) % 4 == 0 && ld_src % 4 == 0 && src_stride % 4 == 0 && ldh % 4 == 0 &&
             aligned16(src) && aligned16(h) && aligned16(norm_w) && aligned16(shift) && aligned16(shift_state) && aligned16(carry);
  if (dst) vec = vec && ld_dst % 4 == 0 && dst_stride % 4 == 0 && aligned16(dst);
  if (y) vec = vec && ldy % 4 == 0 && aligned16(y);
  const size_t lds = ((size_t)(shift ? 2 : 1) * width + (groups > 4 ? groups : 4)) * sizeof(float);
  if (lds > 64 * 1024) return MI_EUNSUPPORTED;
  const int blocks = (rows + per - 1) / per;
  switch (n_streams) {
    case 1: launch_stream<1>(a, vec, blocks, lds, S(stream)); break;
    case 2: launch_stream<2>(a, vec, blocks, lds, S(stream)); break;
    case 3: launch_stream<3>(a, vec, blocks, lds, S(stream)); break;
    case 4: launch_stream<4>(a, vec, blocks, lds, S(stream)); break;
    case 5: launch_stream<5>(a, vec, blocks, lds, S(stream)); break;
    case 6: launch_stream<6>(a, vec, blocks, lds, S(stream)); break;
    case 7: launch_stream<7>(a, vec, blocks, lds, S(stream)); break;
    default: launch_stream<8>(a, vec, blocks, lds, S(stream)); break;
  }
  if (check_launch() != MI_OK) return MI_ELAUNCH;
  if (!several) return MI_OK;
  hipLaunchKernelGGL(stream_carry_kernel, dim3((width + 255) / 256, n_seqs), dim3(256), 0, S(stream), carry, shift_state, cu_q,
                     slot_ids, width);
  return check_launch();
}

extern "C" int mi_diff_heads(const float* o, int64_t ldo_in, const float* lam, int D, float diff, float eps,
                             const float* gate, int64_t ldg, float* out, int64_t ldo, int rows, int H, int G, int Dv,
                             mi_stream stream) {
  if (!o || !lam || !out || rows < 0 || D < 1 || H < 1 || G < 1 || H % G || Dv < 1) return MI_EINVAL;
  if (ldo_in < 2 * (int64_t)H * Dv || ldo < (int64_t)H * Dv || (gate && ldg < H)) return MI_EINVAL;
  if (Dv > 512) return MI_EUNSUPPORTED;
  if (rows == 0) return MI_OK;
#define MI_DIFF(VPL)                                                                                                      \
  hipLaunchKernelGGL((diff_heads_kernel<VPL>), dim3(rows), dim3(256), 0, S(stream), o, ldo_in, lam, D, diff, eps, gate, ldg, \
                     out, ldo, H, G, Dv)
  if (Dv <= 64) MI_DIFF(1);
  else if (Dv <= 128) MI_DIFF(2);
  else if (Dv <= 256) MI_DIFF(4);
  else MI_DIFF(8);
#undef MI_DIFF
  return check_launch();
}

// a head's key channels as the kernel keeps them: padded to 64, 128 or 256
static int gd_pad(int D) { return D <= 64 ? 64 : D <= 128 ? 128 : D <= 256 ? 256 : 0; }

extern "C" int64_t mi_general_delta_state_elems(int H, int D, int Dv) {
  const int dp = gd_pad(D);
  if (H < 1 || D < 1 || Dv < 1 || !dp) return -1;
  return (int64_t)H * ((Dv + kGdCols - 1) / kGdCols) * kGdCols * dp;
}

extern "C" int mi_general_delta(const float* proj, int64_t ld, int r_off, int k_off, int v_off, int a_off,
                                const float* w_decay, int64_t ldw, float* state, const int32_t* cu_q,
                                const int32_t* kv_lens, const int32_t* slot_ids, int n_seqs, int rows, int H, int D, int Dv,
                                float* out, int64_t ldo, mi_stream stream) {
  if (!proj || !w_decay || !state || !cu_q || !kv_lens || !slot_ids || !out || rows < 0 || n_seqs < 1) return MI_EINVAL;
  if (H < 1 || D < 1 || Dv < 1 || ldw < (int64_t)H * D || ldo < (int64_t)H * Dv) return MI_EINVAL;
  for (int off : {r_off, k_off, a_off})
    if (off < 0 || ld < off + (int64_t)H * D) return MI_EINVAL;
  if (v_off < 0 || ld < v_off + (int64_t)H * Dv) return MI_EINVAL;
  const int dp = gd_pad(D), blocks = (Dv + kGdCols - 1) / kGdCols;
  if (!dp || H > 65535 || blocks > 65535) return MI_EUNSUPPORTED;
  if (rows == 0) return MI_OK;
  const dim3 grid(n_seqs, H, blocks);
#define MI_GD(LANES, DR, CPL, ROWS)                                                                                     \
  hipLaunchKernelGGL((general_delta_kernel<LANES, DR, CPL, ROWS>), grid, dim3(LANES * kGdCols / CPL), 0, S(stream), proj, ld, \
                     r_off, k_off, v_off, a_off, w_decay, ldw, state, cu_q, kv_lens, slot_ids, H, D, Dv, out, ldo)
  if (dp == 64) MI_GD(16, 4, 1, 16);
  else if (dp == 128) MI_GD(16, 8, 1, 16);
  else MI_GD(16, 16, 2, 8);
#undef MI_GD
  return check_launch();
}
