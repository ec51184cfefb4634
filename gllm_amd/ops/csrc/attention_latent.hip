// Attention over a paged low-rank latent, gfx950 matrix cores (bf16).
//
// Every token caches ONE row, [latent (R) | rotated key part (Dr)]; all H
// query heads of a token attend to the same rows, and the value is the
// first R columns of the row. So a (token, head) pair is one row of a
// matrix product, and a workgroup takes BQ = 16 RG consecutive pairs of a
// sequence whatever the head count is:
//   score = (q_lat . latent + q_rot . rotated) * scale
//   position i sees 0 <= i - j < window (window <= 0: every j <= i)
//   softmax denominator: sum exp(s) + exp(sink_h)
// One kernel serves prompt portions, mixed batches and decoding; decode-
// only batches split the keys over blockIdx.z and merge with an fp32 pass.
//
// 512 threads = 8 waves, one workgroup per CU at the largest rank. Keys
// stream in tiles of 64 through two LDS slots (global -> LDS loads, the
// next tile in flight while the current one is worked on); the row index
// of a tile's keys comes from the block table one tile earlier still.
//   Q K^T   wave = (row group, key group): 16 rows x 16 NF keys, the query
//           fragments in registers for the whole walk
//   softmax fp32, running max and sum per row; the key groups of a row
//           agree on the max through LDS
//   P V     wave = an eighth of the value columns, all rows: every latent
//           element is read from LDS once, transposed on the way by
//           ds_read_tr16_b64 (4 keys x 16 columns per 16 lanes)
// LDS rows are swizzled in 16 B units so that both access patterns spread
// over the banks (row pitch = 128 B mod 256 B).

#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>
#include "common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) float acc4;
typedef __attribute__((address_space(3))) shortx4 lds_shortx4;

namespace {

constexpr int LA_BLOCK = 512;
constexpr int LA_KEYS = 64;            // keys per tile
constexpr int LA_PT = LA_KEYS + 8;     // padded row of the P tile

DEV_INLINE int la_swz(int row) {
  return ((row & 7) ^ ((row & 8) ? 5 : 0)) << 4;
}

// reductions over the 16 adjacent lanes of a DPP row
#define LA_DPP(v, ctrl)                                                     \
  __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(                    \
      0, __builtin_bit_cast(int, v), ctrl, 0xF, 0xF, true))
DEV_INLINE float row16_max(float v) {
  v = fmaxf(v, LA_DPP(v, 0xB1));   // [1,0,3,2]
  v = fmaxf(v, LA_DPP(v, 0x4E));   // [2,3,0,1]
  v = fmaxf(v, LA_DPP(v, 0x141));  // mirror of each 8
  return fmaxf(v, LA_DPP(v, 0x140));  // mirror of the 16
}
DEV_INLINE float row16_sum(float v) {
  v += LA_DPP(v, 0xB1);
  v += LA_DPP(v, 0x4E);
  v += LA_DPP(v, 0x141);
  return v + LA_DPP(v, 0x140);
}
#undef LA_DPP

struct LatentArgs {
  __hip_bfloat16 *out;   // element (h, t, d) at h * out_hs + t * out_ts + d
  long out_hs, out_ts;
  float *part_o;         // [splits, T * H, R]   (SPLIT)
  float *part_lse;       // [splits, T * H]
  const __hip_bfloat16 *q_lat;
  long ql_hs, ql_ts;
  const __hip_bfloat16 *q_rot;
  long qr_hs, qr_ts;
  const __hip_bfloat16 *cache;  // [pages * page, R + Dr]
  const int *block_table;
  int bt_stride;
  const int *seq_lens, *qsl;
  const float *sinks;    // [H] or null
  int page, H, R, Dr, window, splits;
  long rows_total;       // T * H
  float scale;
};

// KT: 32-wide steps over R + Dr (even); NTW: 16-wide value tiles per wave;
// RG: row groups of 16 (token, head) pairs per workgroup (1, 2 or 4)
template <int KT, int NTW, int RG, bool SPLIT>
__global__ __launch_bounds__(LA_BLOCK, 2) void latent_attention_kernel(
    LatentArgs a) {
  constexpr int BQ = 16 * RG;
  constexpr int NF = RG == 4 ? 2 : 1;     // key fragments per wave
  constexpr int NK = 4 / NF;              // key groups
  constexpr int ROW_B = KT * 64;          // LDS row bytes
  constexpr int TILE_B = LA_KEYS * ROW_B;
  constexpr int GL = TILE_B / 1024 / 8;   // 1 KiB loads per wave and tile
  static_assert(TILE_B % 8192 == 0, "whole loads per wave");
  __shared__ __attribute__((aligned(16))) char kbuf[2 * TILE_B];
  __shared__ __attribute__((aligned(16))) __hip_bfloat16 pt[BQ * LA_PT];
  __shared__ __attribute__((aligned(16))) float s_alpha[BQ];
  __shared__ float s_max[NK][BQ];
  __shared__ int s_row[LA_KEYS];

  const int tile = blockIdx.x, b = blockIdx.y, split = blockIdx.z;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int l16 = lane & 15, lhi = lane >> 4;
  const int H = a.H, R = a.R, D = a.R + a.Dr;
  const int q_start = a.qsl[b], q_len = a.qsl[b + 1] - q_start;
  const int rows = q_len * H;
  if (tile * BQ >= rows) return;
  const int past = a.seq_lens[b] - q_len;
  const int tok0 = tile * BQ / H;
  const int tok1 = min(rows - 1, tile * BQ + BQ - 1) / H;
  // keys any row of this workgroup sees, then this split's share of them
  int kv_hi = past + tok1 + 1;
  int kv_lo = a.window > 0 ? max(0, past + tok0 - a.window + 1) : 0;
  const long row0 = (long)q_start * H + (long)tile * BQ;
  if (SPLIT) {
    const int per = ((kv_hi - kv_lo + LA_KEYS - 1) / LA_KEYS + a.splits - 1) /
                    a.splits * LA_KEYS;
    kv_lo += split * per;
    kv_hi = min(kv_hi, kv_lo + per);
    if (kv_lo >= kv_hi) {  // nothing left for this split
      for (int r = tid; r < BQ; r += LA_BLOCK)
        if (tile * BQ + r < rows)
          a.part_lse[(long)split * a.rows_total + row0 + r] = -INFINITY;
      return;
    }
  }
  const int span = a.window > 0 ? a.window : 0x7fffffff;
  const int n_tiles = (kv_hi - kv_lo + LA_KEYS - 1) / LA_KEYS;
  const int *bt = a.block_table + (long)b * a.bt_stride;

  const int rg = RG == 4 ? wave & 3 : RG == 2 ? wave & 1 : 0;
  const int kq = RG == 4 ? wave >> 2 : RG == 2 ? wave >> 1 : wave;
  const bool scores = kq < NK;  // this wave forms scores (RG 1: half do)

  // key n of a tile (past the end: the last key again, its scores masked)
  auto key_at = [&](int t, int n) {
    return min(kv_lo + t * LA_KEYS + n, kv_hi - 1);
  };
  // 1 KiB per wave and load, straight into LDS; a lane whose column lies
  // past the row (padding) re-reads the row's start: finite, times a zero
  // query element. Issued as inline assembly: the loop orders these loads
  // against the LDS reads itself (vmcnt, then the barrier), and the
  // compiler must not wait for the next tile ahead of this tile's reads.
  // (row << 16 | byte column) of this lane's place in load j, kept packed:
  // decoded per use, or the loop would carry 3 GL address registers.
  int place[GL];
#pragma unroll
  for (int j = 0; j < GL; ++j) {
    const int p = (wave * GL + j) * 1024 + lane * 16;
    const int row = p / ROW_B;
    const int col = (p % ROW_B) ^ la_swz(row);
    place[j] = row << 16 | (col < D * 2 ? col : 0);
  }
  const unsigned k_lds =
      (unsigned)(unsigned long)(__attribute__((address_space(3))) char *)kbuf +
      wave * GL * 1024;
  auto stage = [&](int t) {
    const unsigned base = k_lds + (t & 1) * TILE_B;
#pragma unroll
    for (int j = 0; j < GL; ++j) {
      int pl = place[j];
      asm volatile("" : "+v"(pl));
      const char *src = reinterpret_cast<const char *>(a.cache) +
                        (long)s_row[pl >> 16] * (D * 2) +
                        (pl & 0xffff);
      asm volatile(
          "s_mov_b32 m0, %1\n\t"
          "s_nop 0\n\t"
          "global_load_lds_dwordx4 %0, off"
          :
          : "v"(src), "s"(__builtin_amdgcn_readfirstlane(base + j * 1024))
          : "memory", "m0");
    }
  };

  int page_id = 0;  // block-table entry of this thread's key, next tile
  if (tid < LA_KEYS) {
    const int j = key_at(0, tid);
    s_row[tid] = bt[j / a.page] * a.page + j % a.page;
    page_id = bt[key_at(1, tid) / a.page];
  }
  // query fragments: row rg * 16 + l16, columns kt * 32 + lhi * 8
  bf16x8 qf[KT];
  {
    const int rr = tile * BQ + rg * 16 + l16;
    const bool ok = scores && rr < rows;
    const long t = q_start + (ok ? rr / H : 0);
    const int h = ok ? rr % H : 0;
    const __hip_bfloat16 *ql = a.q_lat + h * a.ql_hs + t * a.ql_ts;
    const __hip_bfloat16 *qr = a.q_rot + h * a.qr_hs + t * a.qr_ts;
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const int c = kt * 32 + lhi * 8;
      if (ok && c < R)
        qf[kt] = *reinterpret_cast<const bf16x8 *>(ql + c);
      else if (ok && c < D)
        qf[kt] = *reinterpret_cast<const bf16x8 *>(qr + (c - R));
      else
        qf[kt] = bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
    }
  }
  // this lane's four rows: position, running max, its share of the sum
  int qpos[4];
  float m_run[4], l_run[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int rr = min(tile * BQ + rg * 16 + lhi * 4 + r, rows - 1);
    qpos[r] = past + rr / H;
    m_run[r] = -INFINITY;
    l_run[r] = 0.f;
    if (!SPLIT && a.sinks) {  // a key already seen, without a value
      m_run[r] = a.sinks[rr % H];
      l_run[r] = (kq == 0 && l16 == 0) ? 1.f : 0.f;
    }
  }
  acc4 o[RG][NTW];
#pragma unroll
  for (int g = 0; g < RG; ++g)
#pragma unroll
    for (int n = 0; n < NTW; ++n) o[g][n] = acc4{0.f, 0.f, 0.f, 0.f};

  // what the loop reads from registers has arrived before it starts (a
  // load still pending here would make the loop wait for its own tiles)
#pragma unroll
  for (int kt = 0; kt < KT; ++kt) asm volatile("" : "+v"(qf[kt]));
#pragma unroll
  for (int r = 0; r < 4; ++r) asm volatile("" : "+v"(m_run[r]));
  asm volatile("" : "+v"(page_id));
  __syncthreads();
  stage(0);

  for (int it = 0; it < n_tiles; ++it) {
    const int kv0 = kv_lo + it * LA_KEYS;
    const char *kt_lds = kbuf + (it & 1) * TILE_B;
    // every wave's loads of this tile have landed; and every wave is done
    // with the other slot, which the next tile goes to
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    if (tid < LA_KEYS && it + 1 < n_tiles)
      s_row[tid] = page_id * a.page + key_at(it + 1, tid) % a.page;
    __syncthreads();
    if (tid < LA_KEYS && it + 2 < n_tiles)
      page_id = bt[key_at(it + 2, tid) / a.page];
    if (it + 1 < n_tiles) stage(it + 1);

    acc4 s[NF];
    if (scores) {
#pragma unroll
      for (int f = 0; f < NF; ++f) s[f] = acc4{0.f, 0.f, 0.f, 0.f};
      // (the swizzle depends on l16 only and moves a column inside its
      // 128 B block: two offsets serve all steps)
      const char *kbase = kt_lds + (kq * NF * 16 + l16) * ROW_B;
      const int col[2] = {(lhi * 16) ^ la_swz(l16),
                          (64 + lhi * 16) ^ la_swz(l16)};
#pragma unroll
      for (int kt = 0; kt < KT; ++kt)
#pragma unroll
        for (int f = 0; f < NF; ++f) {
          const bf16x8 kf = *reinterpret_cast<const bf16x8 *>(
              kbase + col[kt & 1] + (f * 16 * ROW_B + (kt >> 1) * 128));
          s[f] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[kt], kf, s[f], 0,
                                                         0, 0);
        }
      const bool inside =
          kv0 + LA_KEYS - 1 <= past + tok0 && kv0 + LA_KEYS <= kv_hi &&
          (a.window <= 0 || past + tok1 - kv0 < a.window);
#pragma unroll
      for (int f = 0; f < NF; ++f)
#pragma unroll
        for (int r = 0; r < 4; ++r) s[f][r] *= a.scale;
      if (!inside) {
#pragma unroll
        for (int f = 0; f < NF; ++f) {
          const int j = kv0 + (kq * NF + f) * 16 + l16;
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int dist = qpos[r] - j;
            const bool out = dist < 0 || dist >= span || j >= kv_hi;
            s[f][r] = out ? -INFINITY : s[f][r];
          }
        }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float mx = s[0][r];
#pragma unroll
        for (int f = 1; f < NF; ++f) mx = fmaxf(mx, s[f][r]);
        mx = row16_max(mx);
        if (l16 == 0) s_max[kq][rg * 16 + lhi * 4 + r] = mx;
      }
    }
    __syncthreads();
    if (scores) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = rg * 16 + lhi * 4 + r;
        float mn = m_run[r];
#pragma unroll
        for (int g = 0; g < NK; ++g) mn = fmaxf(mn, s_max[g][row]);
        const float base = mn == -INFINITY ? 0.f : mn;
        const float alpha = __expf(m_run[r] - base);
        m_run[r] = mn;
        float sum = 0.f;
#pragma unroll
        for (int f = 0; f < NF; ++f) {
          const float p = __expf(s[f][r] - base);
          sum += p;
          pt[row * LA_PT + (kq * NF + f) * 16 + l16] = __float2bfloat16(p);
        }
        l_run[r] = l_run[r] * alpha + sum;
        if (kq == 0 && l16 == 0) s_alpha[row] = alpha;
      }
    }
    __syncthreads();

    // O <- diag(alpha) O + P V, this wave's value columns
#pragma unroll
    for (int g = 0; g < RG; ++g) {
      const acc4 al =
          *reinterpret_cast<const acc4 *>(&s_alpha[g * 16 + lhi * 4]);
#pragma unroll
      for (int n = 0; n < NTW; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[g][n][r] *= al[r];
    }
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      bf16x8 pf[RG];
#pragma unroll
      for (int g = 0; g < RG; ++g)
        pf[g] = *reinterpret_cast<const bf16x8 *>(
            &pt[(g * 16 + l16) * LA_PT + ks * 32 + lhi * 8]);
#pragma unroll
      for (int n = 0; n < NTW; ++n) {
        // keys ks * 32 + lhi * 8 + 0..7 of column c0 + l16: two transposed
        // reads of 4 keys, lane l16 addressing key l16 / 4, columns
        // c0 + 4 (l16 % 4) .. + 3
        const int cb = ((wave * NTW + n) * 16 + (l16 & 3) * 4) * 2;
        const int k0 = lhi * 8 + (l16 >> 2);
        const char *p0 = kt_lds + ks * 32 * ROW_B + k0 * ROW_B +
                         (cb & ~127) + ((cb & 112) ^ la_swz(k0)) + (cb & 15);
        const char *p1 = kt_lds + ks * 32 * ROW_B + (k0 + 4) * ROW_B +
                         (cb & ~127) + ((cb & 112) ^ la_swz(k0 + 4)) +
                         (cb & 15);
        union {
          shortx4 h[2];
          bf16x8 v;
        } vf;
        vf.h[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (lds_shortx4 *)const_cast<char *>(p0));
        vf.h[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (lds_shortx4 *)const_cast<char *>(p1));
#pragma unroll
        for (int g = 0; g < RG; ++g)
          o[g][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[g], vf.v,
                                                            o[g][n], 0, 0, 0);
      }
    }
  }

  // row sums: lanes of a row, then key groups
  __syncthreads();  // s_max / s_alpha are free
  if (scores) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = rg * 16 + lhi * 4 + r;
      const float l = row16_sum(l_run[r]);
      if (l16 == 0) {
        s_max[kq][row] = l;
        if (kq == 0) s_alpha[row] = m_run[r];
      }
    }
  }
  __syncthreads();
#pragma unroll
  for (int g = 0; g < RG; ++g)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = g * 16 + lhi * 4 + r;
      const int rr = tile * BQ + row;
      if (rr >= rows) continue;
      float l = 0.f;
#pragma unroll
      for (int k = 0; k < NK; ++k) l += s_max[k][row];
      const float inv = l > 0.f ? 1.f / l : 0.f;
      if (SPLIT) {
        const long prow = (long)split * a.rows_total + row0 + row;
#pragma unroll
        for (int n = 0; n < NTW; ++n) {
          const int d = (wave * NTW + n) * 16 + l16;
          if (d < R) a.part_o[prow * R + d] = o[g][n][r] * inv;
        }
        if (wave == 0 && l16 == 0)
          a.part_lse[prow] =
              l > 0.f ? s_alpha[row] + __logf(l) : -INFINITY;
      } else {
        __hip_bfloat16 *dst =
            a.out + (rr % H) * a.out_hs + (q_start + rr / H) * a.out_ts;
#pragma unroll
        for (int n = 0; n < NTW; ++n) {
          const int d = (wave * NTW + n) * 16 + l16;
          if (d < R) dst[d] = __float2bfloat16(o[g][n][r] * inv);
        }
      }
    }
}

// one workgroup per (token, head): weights exp(lse) of the splits, the
// sink joining the denominator. grid (T * H), block 128; splits <= 32.
__global__ __launch_bounds__(128) void latent_merge_kernel(LatentArgs a) {
  __shared__ float wt[32];
  const long row = blockIdx.x;
  const int h = row % a.H;
  const long t = row / a.H;
  if (threadIdx.x < WAVE_SIZE) {
    const int s = threadIdx.x;
    const float lse =
        s < a.splits ? a.part_lse[(long)s * a.rows_total + row] : -INFINITY;
    const float sink = a.sinks ? a.sinks[h] : -INFINITY;
    const float mx = fmaxf(wave_reduce_max(lse), sink);
    const float w = __expf(lse - mx);  // 0: that split wrote nothing
    const float den = wave_reduce_sum(w) + __expf(sink - mx);
    if (s < 32) wt[s] = w / den;
  }
  __syncthreads();
  __hip_bfloat16 *dst = a.out + h * a.out_hs + t * a.out_ts;
  const float *src = a.part_o + row * a.R;
  const long step = a.rows_total * a.R;
  for (int d = threadIdx.x * 4; d < a.R; d += 512) {
    acc4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int s = 0; s < a.splits; ++s) {
      const float w = wt[s];
      if (w > 0.f) {
        const acc4 v = *reinterpret_cast<const acc4 *>(src + s * step + d);
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] += w * v[e];
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) dst[d + e] = __float2bfloat16(o[e]);
  }
}

template <int KT, int NTW>
void launch_latent(LatentArgs a, int B, int rg, int tiles, bool split,
                   hipStream_t stream) {
  const dim3 grid(tiles, B, split ? a.splits : 1);
#define GO(RGV, SP)                                                         \
  hipLaunchKernelGGL((latent_attention_kernel<KT, NTW, RGV, SP>), grid,     \
                     dim3(LA_BLOCK), 0, stream, a)
  if (split) {
    if (rg == 1) GO(1, true);
    else if (rg == 2) GO(2, true);
    else GO(4, true);
  } else {
    if (rg == 1) GO(1, false);
    else if (rg == 2) GO(2, false);
    else GO(4, false);
  }
#undef GO
}

}  // namespace

// false = this geometry has no instance (the caller takes the generic
// kernel); nothing has been launched then
bool latent_attention_mfma(torch::Tensor out, torch::Tensor q_lat,
                           torch::Tensor q_rot, torch::Tensor cache,
                           torch::Tensor block_table, torch::Tensor seq_lens,
                           torch::Tensor query_start_loc, double scale,
                           long window, c10::optional<torch::Tensor> sinks,
                           long max_query_len) {
  const long H = q_lat.size(0), T = q_lat.size(1), R = q_lat.size(2);
  const long Dr = q_rot.size(2), D = R + Dr;
  if (q_lat.scalar_type() != at::kBFloat16) return false;
  if (R % 8 || Dr % 8 || R > 512) return false;
  const int bucket = (R <= 128 && D <= 192)   ? 0
                     : (R <= 256 && D <= 320) ? 1
                     : D <= 576               ? 2
                                              : -1;
  if (bucket < 0) return false;
  auto on16 = [](const torch::Tensor &t) {
    return reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0 &&
           t.stride(0) % 8 == 0 && t.stride(1) % 8 == 0 && t.stride(2) == 1;
  };
  if (T == 0) return true;
  if (!on16(q_lat) || (Dr && !on16(q_rot))) return false;
  TORCH_CHECK(q_lat.is_cuda() && q_rot.scalar_type() == at::kBFloat16 &&
              q_rot.size(0) == T && q_rot.size(1) == H);
  TORCH_CHECK(out.dim() == 3 && out.sizes() == q_lat.sizes() &&
              out.scalar_type() == at::kBFloat16 && out.stride(2) == 1);
  TORCH_CHECK(cache.is_contiguous() && cache.dim() == 4 &&
              cache.scalar_type() == at::kBFloat16 && cache.size(2) == 1 &&
              cache.size(3) == D &&
              reinterpret_cast<uintptr_t>(cache.data_ptr()) % 16 == 0,
              "latent cache: [pages, page, 1, rank + rotated]");
  TORCH_CHECK(cache.size(0) * cache.size(1) < (1L << 31));
  TORCH_CHECK(block_table.scalar_type() == at::kInt &&
              block_table.dim() == 2 && block_table.stride(1) == 1);
  TORCH_CHECK(seq_lens.scalar_type() == at::kInt && seq_lens.is_contiguous());
  TORCH_CHECK(query_start_loc.scalar_type() == at::kInt &&
              query_start_loc.is_contiguous());
  const int B = seq_lens.numel();
  TORCH_CHECK(query_start_loc.numel() >= B + 1 && block_table.size(0) >= B);
  TORCH_CHECK(max_query_len >= 1 && max_query_len * H < (1L << 31) &&
              T * H < (1L << 31));
  LatentArgs a{};
  a.out = (__hip_bfloat16 *)out.data_ptr();
  a.out_hs = out.stride(0);
  a.out_ts = out.stride(1);
  a.q_lat = (const __hip_bfloat16 *)q_lat.data_ptr();
  a.ql_hs = q_lat.stride(0);
  a.ql_ts = q_lat.stride(1);
  a.q_rot = (const __hip_bfloat16 *)q_rot.data_ptr();
  a.qr_hs = q_rot.stride(1);
  a.qr_ts = q_rot.stride(0);
  a.cache = (const __hip_bfloat16 *)cache.data_ptr();
  a.block_table = block_table.data_ptr<int>();
  a.bt_stride = block_table.stride(0);
  a.seq_lens = seq_lens.data_ptr<int>();
  a.qsl = query_start_loc.data_ptr<int>();
  if (sinks.has_value()) {
    TORCH_CHECK(sinks->scalar_type() == at::kFloat && sinks->is_contiguous() &&
                sinks->numel() == H, "sinks: fp32 [H]");
    a.sinks = sinks->data_ptr<float>();
  }
  a.page = cache.size(1);
  a.H = H;
  a.R = R;
  a.Dr = Dr;
  a.window = window > 0 ? (int)std::min<long>(window, 1L << 30) : 0;
  a.rows_total = T * H;
  a.scale = scale;
  const long rows = max_query_len * H;  // pairs of the longest portion
  const int rg = rows <= 16 ? 1 : rows <= 32 ? 2 : 4;
  const int tiles = (rows + 16 * rg - 1) / (16 * rg);
  // decode-only: enough workgroups for the chip, however many keys each
  // sequence turns out to have (a captured launch serves every length)
  int splits = 1;
  if (max_query_len == 1) {
    const long most = a.window ? (a.window + LA_KEYS - 1) / LA_KEYS : 64;
    while (splits < 32 && (long)B * tiles * splits < 256 &&
           splits * 2 <= most)
      splits *= 2;
  }
  a.splits = splits;
  torch::Tensor part, lse;
  if (splits > 1) {
    auto opt = out.options().dtype(at::kFloat);
    part = torch::empty({splits, T * H, R}, opt);
    lse = torch::empty({splits, T * H}, opt);
    a.part_o = part.data_ptr<float>();
    a.part_lse = lse.data_ptr<float>();
  }
  auto stream = at::cuda::getCurrentCUDAStream();
  if (bucket == 0) launch_latent<6, 1>(a, B, rg, tiles, splits > 1, stream);
  else if (bucket == 1) launch_latent<10, 2>(a, B, rg, tiles, splits > 1, stream);
  else launch_latent<18, 4>(a, B, rg, tiles, splits > 1, stream);
  HIP_CHECK_KERNEL();
  if (splits > 1) {
    hipLaunchKernelGGL(latent_merge_kernel, dim3(T * H), dim3(128), 0, stream,
                       a);
    HIP_CHECK_KERNEL();
  }
  return true;
}
