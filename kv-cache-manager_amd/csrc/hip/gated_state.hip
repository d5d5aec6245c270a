// Two recurrences whose state is a matrix per head that decays by one number per head and token, S [dk, dv]:
//
//   delta 1 (the gated delta rule)    g = exp(-exp(a_log) softplus(a + dt_bias)),  beta = sigmoid(b)
//       q <- q / sqrt(|q|^2 + 1e-6) * dk^(-1/2),  k <- k / sqrt(|k|^2 + 1e-6)
//       S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//   delta 0 (state-space duality)     dt = softplus(a + dt_bias)
//       S <- exp(-exp(a_log) dt) S + dt k v^T;  o = S^T q + d_skip v
//   delta 0 with `decay` (a fixed decay per head)     q, k, v <- silu of what is given, where asked for
//       S <- decay S + k v^T;  o = S^T q
//
// q and k come in `groups` heads of dk entries, v in `heads` heads of dv; head h reads group h / (heads / groups).  Everything
// here is 32-bit.  A run that starts at position 0 starts from zero without reading its slot.
//
// The walk takes one token after another.  A value column j of S needs S^T k of its own column only, so columns are spread
// over lanes and workgroups (JPT * 256 / G of them a workgroup, the key dimension of a column over G lanes, JPT columns a lane,
// so that a staged q and k serve JPT columns; a column's operations do not depend on JPT); the tokens' vectors
// are staged through LDS a few at a time, the next ones requested before the current are computed, and a token's scalars
// (decay, rate, the lengths of its q and k) are made as its vectors are staged, so that no transcendental function and no
// sum across the head sits in the chain from token to token.
//
// Long runs are walked in pieces of L rows, all pieces at once.  A piece maps the state that enters it to the state that
// leaves it by S -> A S + B (both recurrences are linear in S): B is the piece walked from zero, A is the product of its
// decays, or, for the delta rule, the dk x dk matrix that the same walk makes of the identity when its values are zero: dk
// further columns beside the dv.  Three launches: every piece's A and B; the states that enter the pieces, one after another
// (a small product each); every piece again from the state that enters it, now with outputs.
#include "common.h"
#include "kvcm_hip.h"

namespace kvcm {

__device__ __forceinline__ float softplus32(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

struct StateArgs {
  const float *q, *k, *v, *a, *b;      // 32-bit rows
  int ldq, ldk, ldv, lda, ldb;
  const float *dt_bias, *a_log, *d_skip;
  const float* decay;                  // [heads]: a fixed decay (a, dt_bias, a_log, d_skip are not read)
  int silu_in;
  float* o;
  int ldo;
  float* state;                        // [slots, heads, dk, dv]
  const int *run_start, *seq_start, *state_slots;
  int heads, groups, dk, dv, col_blocks;
  float* carry;                        // pieces: per (piece, head) [dk][W] with W = dv + dk (delta) or dv, then per (piece, head) the decay
  int piece, pieces_per_seq, total_pieces;
};

// which rows of sequence s piece number p covers, and where its carry lies (pieces of all sequences are numbered so that no
// two meet: a sequence starts at floor(its first row / piece) + its own number)
__device__ __forceinline__ int piece_place(int run0, int s, int p, int piece) { return run0 / piece + s + p; }

// ENDS: the first of the three launches (no outputs, a state of W columns from zero / identity, written to the carry)
template <int DKP, int G, int JPT, int TILE, bool DELTA, bool ENDS>
__global__ void __launch_bounds__(256) gated_state_kernel(StateArgs A) {
  constexpr int IPT = DKP / G, LC = 256 / G, CB = LC * JPT, KAT = ENDS ? 0 : DKP, V = KAT + DKP + CB, SC = 4;
  constexpr int PF = (TILE * V + 255) / 256;
  __shared__ __attribute__((aligned(16))) float tile[TILE][V + SC];      // per token: q (not without outputs), k (zero beyond dk), v of these columns, scalars
  const int head = blockIdx.x / A.col_blocks, cb = blockIdx.x % A.col_blocks;
  const int s = blockIdx.y / A.pieces_per_seq, p = blockIdx.y % A.pieces_per_seq;
  const int dk = A.dk, dv = A.dv, W = ENDS && DELTA ? dv + dk : dv;
  const int g = threadIdx.x % G, jl = threadIdx.x / G, j0 = cb * CB + jl;      // this lane's columns: j0 + c * LC, c < JPT
  int r0 = A.run_start[s], r1 = A.run_start[s + 1];
  const int slot = A.state_slots[s];
  const int run0 = r0, run1 = r1;
  const bool pieces = A.piece > 0;
  if (pieces) {
    r0 = run0 + p * A.piece;
    r1 = run1 - r0 < A.piece ? run1 : r0 + A.piece;
  }
  if (r1 <= r0) return;
  const bool last = r1 == run1;
  if (ENDS && (last || slot < 0)) return;      // nothing follows the last piece
  if (slot < 0) {
    if (g == 0)
      for (int row = r0; row < r1; ++row)
        for (int c = 0; c < JPT; ++c)
          if (j0 + c * LC < dv) A.o[size_t(row) * A.ldo + size_t(head) * dv + j0 + c * LC] = 0.f;
    return;
  }
  const int group = head / (A.heads / A.groups);
  const bool fresh = A.seq_start[s] == 0;
  float* st = A.state + ((size_t(slot) * A.heads + head) * dk) * dv;                        // [i][j]
  const int CW = DELTA ? dv + dk : dv;                                                       // a carry's columns
  float* cst = nullptr;
  if (pieces) cst = A.carry + ((size_t(piece_place(run0, s, p, A.piece)) * A.heads + head) * dk) * CW;
  float S[JPT][IPT];
#pragma unroll
  for (int c = 0; c < JPT; ++c)
#pragma unroll
    for (int il = 0; il < IPT; ++il) {
      const int i = g * IPT + il, j = j0 + c * LC;
      const bool mine = i < dk && j < W;
      if constexpr (ENDS) S[c][il] = (DELTA && mine && j - dv == i) ? 1.f : 0.f;
      else if (pieces) S[c][il] = mine ? cst[size_t(i) * CW + j] : 0.f;
      else S[c][il] = (mine && !fresh) ? st[size_t(i) * dv + j] : 0.f;
    }
  const bool fixed = !DELTA && A.decay;
  const float rate = fixed ? 0.f : -expf(A.a_log[head]), dtb = fixed ? 0.f : A.dt_bias[head];
  const float skip = DELTA || fixed ? 0.f : A.d_skip[head], fixed_keep = fixed ? A.decay[head] : 0.f;
  const float q_scale = 1.0f / sqrtf(float(dk));
  float pf[PF], sa = 0.f, sb = 0.f;
  auto request = [&](int t0) {      // unconditional loads from clamped places, masked afterwards
#pragma unroll
    for (int n = 0; n < PF; ++n) {
      const int e = threadIdx.x + n * 256;
      const int t = e / V, off = e % V;
      const int row = t0 + t < r1 ? t0 + t : r1 - 1;
      const bool vec = off < KAT + DKP;
      const int i = off % DKP, jj = cb * CB + (off - KAT - DKP);
      const bool ok = t < TILE && t0 + t < r1 && (vec ? i < dk : jj < dv);
      const size_t col = size_t(group) * dk + (i < dk ? i : dk - 1);
      const size_t vcol = size_t(head) * dv + ((jj >= 0 && jj < dv) ? jj : 0);
      const float* src = !vec ? A.v + size_t(row) * A.ldv + vcol : off < KAT ? A.q + size_t(row) * A.ldq + col : A.k + size_t(row) * A.ldk + col;
      const float val = *src;
      pf[n] = ok ? val : 0.f;
    }
    const int t = threadIdx.x < TILE ? threadIdx.x : TILE - 1;
    const int row = t0 + t < r1 ? t0 + t : r1 - 1;
    if (!fixed) sa = A.a[size_t(row) * A.lda + head];
    if constexpr (DELTA) sb = A.b[size_t(row) * A.ldb + head];
  };
  auto stage = [&]() {
#pragma unroll
    for (int n = 0; n < PF; ++n) {
      const int e = threadIdx.x + n * 256;
      if (e < TILE * V) tile[e / V][e % V] = !DELTA && A.silu_in ? silu<bf16_t>(pf[n]) : pf[n];      // (silu(0) = 0: what was masked stays 0)
    }
    if (threadIdx.x < TILE) {
      const float dt = softplus32(sa + dtb);
      tile[threadIdx.x][V] = fixed ? fixed_keep : expf(rate * dt);
      tile[threadIdx.x][V + 1] = DELTA ? 1.0f / (1.0f + expf(-sb)) : fixed ? 1.f : dt;
    }
    if constexpr (DELTA) {      // the lengths of the staged q and k: sixteen lanes a vector
      __syncthreads();
      const int vec = threadIdx.x / 16, l = threadIdx.x % 16;
      if (ENDS ? vec < TILE : vec < 2 * TILE) {
        const int t = ENDS ? vec : vec / 2;
        const bool key = ENDS || (vec & 1);
        const float* x = &tile[t][key ? KAT : 0];
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < DKP / 16; ++i) ss = fmaf(x[l + i * 16], x[l + i * 16], ss);
        ss = group_sum<16>(ss);
        if (l == 0) tile[t][V + 2 + (key ? 1 : 0)] = (1.0f / sqrtf(ss + 1e-6f)) * (key ? 1.0f : q_scale);
      }
    }
  };
  float decay = 1.f;
  request(r0);
  stage();
  __syncthreads();
  for (int t0 = r0; t0 < r1; t0 += TILE) {
    const int nt = r1 - t0 < TILE ? r1 - t0 : TILE;
    const bool more = t0 + TILE < r1;
    if (more) request(t0 + TILE);
    for (int t = 0; t < nt; ++t) {
      const float* tv = tile[t];
      const float keep = tv[V], take = tv[V + 1];
      float kd[IPT], vj[JPT], u[JPT];
#pragma unroll
      for (int il = 0; il < IPT; ++il) kd[il] = tv[KAT + g * IPT + il];
#pragma unroll
      for (int c = 0; c < JPT; ++c) vj[c] = tv[KAT + DKP + c * LC + jl];
      if constexpr (DELTA) {
        const float fk = tv[V + 3];
#pragma unroll
        for (int c = 0; c < JPT; ++c) {
          float sk = 0.f;
#pragma unroll
          for (int il = 0; il < IPT; ++il) {
            S[c][il] *= keep;
            sk = fmaf(kd[il], S[c][il], sk);
          }
          u[c] = sk;
        }
#pragma unroll
        for (int c = 0; c < JPT; ++c) u[c] = take * (vj[c] - group_sum<G>(u[c]) * fk) * fk;
      } else {
#pragma unroll
        for (int c = 0; c < JPT; ++c) {
          u[c] = take * vj[c];
#pragma unroll
          for (int il = 0; il < IPT; ++il) S[c][il] *= keep;
        }
        if constexpr (ENDS) decay *= keep;
      }
      float acc[JPT];
#pragma unroll
      for (int c = 0; c < JPT; ++c) acc[c] = 0.f;
#pragma unroll
      for (int il = 0; il < IPT; ++il) {
        const float qd = ENDS ? 0.f : tv[g * IPT + il];
#pragma unroll
        for (int c = 0; c < JPT; ++c) {
          S[c][il] = fmaf(kd[il], u[c], S[c][il]);
          if constexpr (!ENDS) acc[c] = fmaf(S[c][il], qd, acc[c]);
        }
      }
      if constexpr (!ENDS) {
#pragma unroll
        for (int c = 0; c < JPT; ++c) {
          const float sum = group_sum<G>(acc[c]);
          const int j = j0 + c * LC;
          if (j < dv && g == 0) A.o[size_t(t0 + t) * A.ldo + size_t(head) * dv + j] = DELTA ? sum * tv[V + 2] : fmaf(skip, vj[c], sum);
        }
      }
    }
    __syncthreads();
    if (more) stage();
    __syncthreads();
  }
  if constexpr (ENDS) {
#pragma unroll
    for (int c = 0; c < JPT; ++c)
#pragma unroll
      for (int il = 0; il < IPT; ++il) {
        const int i = g * IPT + il, j = j0 + c * LC;
        if (i < dk && j < W) cst[size_t(i) * CW + j] = S[c][il];
      }
    if (!DELTA && cb == 0 && threadIdx.x == 0)
      A.carry[size_t(A.total_pieces) * A.heads * dk * CW + size_t(piece_place(run0, s, p, A.piece)) * A.heads + head] = decay;
  } else if (last) {
#pragma unroll
    for (int c = 0; c < JPT; ++c)
#pragma unroll
      for (int il = 0; il < IPT; ++il) {
        const int i = g * IPT + il, j = j0 + c * LC;
        if (i < dk && j < W) st[size_t(i) * dv + j] = S[c][il];
      }
  }
}

// the states that enter a sequence's pieces, walked from its slot (or zero): carry[piece].B <- S, then S <- A S + B.
// grid (heads * column blocks of 16, sequences), four lanes a row of S with four columns each; S of these columns in LDS.
// What a step of the walk reads (the row's part of B, the row of A a stretch at a time) does not depend on the state, so it is
// requested a stretch ahead (WIDE: sizes in multiples of four, rows of A read 16 bytes at a time; otherwise as it is used).
constexpr int kPassCols = 16;
template <int DKP, bool DELTA, bool WIDE>
__global__ void __launch_bounds__(DKP * 4) gated_state_pass_kernel(StateArgs A) {
  constexpr int NB = DKP <= 64 ? 16 : 8;                        // 16-byte pieces of a row of A on their way at once
  constexpr int STRETCHES = DELTA ? DKP / 4 / NB : 1;
  __shared__ __attribute__((aligned(16))) float cur[2][DKP][kPassCols];
  const int head = blockIdx.x / A.col_blocks, cb = blockIdx.x % A.col_blocks, s = blockIdx.y;
  const int dk = A.dk, dv = A.dv, CW = DELTA ? dv + dk : dv;
  const int run0 = A.run_start[s], len = A.run_start[s + 1] - run0, slot = A.state_slots[s];
  if (len <= 0 || slot < 0) return;
  const int n = (len + A.piece - 1) / A.piece;
  const int jl = (threadIdx.x % 4) * 4, j0 = cb * kPassCols + jl, i = threadIdx.x / 4, ic = i < dk ? i : dk - 1;
  const bool fresh = A.seq_start[s] == 0;
  const float* st = A.state + (size_t(slot) * A.heads + head) * dk * dv;
  const float* decays = A.carry + size_t(A.total_pieces) * A.heads * dk * CW;
  auto place = [&](int p) { return size_t(piece_place(run0, s, p, A.piece)) * A.heads + head; };
  auto row_of = [&](int p) { return A.carry + (place(p) * dk + ic) * CW; };
  float4 a[NB];
  float b[4], keep = 0.f;
  auto request_a = [&](int p, int stretch) {
    if constexpr (DELTA && WIDE) {
      const float* src = row_of(p) + dv;
#pragma unroll
      for (int q = 0; q < NB; ++q) {
        const int m = (stretch * NB + q) * 4;
        a[q] = *reinterpret_cast<const float4*>(src + (m < dk ? m : 0));
      }
    }
  };
  auto request_b = [&](int p) {
    const float* src = row_of(p);
#pragma unroll
    for (int c = 0; c < 4; ++c) b[c] = src[j0 + c < dv ? j0 + c : dv - 1];
    if constexpr (!DELTA) keep = decays[place(p)];
  };
  // rows of S beyond dk stay zero: what a row of A multiplies there adds nothing
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    cur[0][i][jl + c] = (fresh || i >= dk || j0 + c >= dv) ? 0.f : st[size_t(i) * dv + j0 + c];
    cur[1][i][jl + c] = 0.f;
  }
  if (n > 1) {
    request_b(0);
    request_a(0, 0);
  }
  __syncthreads();
  int now = 0;
  for (int p = 0; p < n; ++p, now ^= 1) {
    const float4 mine = *reinterpret_cast<const float4*>(&cur[now][i][jl]);
    if (p + 1 < n) {
      float acc[4] = {b[0], b[1], b[2], b[3]};
      if constexpr (DELTA) {
        if (p + 2 < n) request_b(p + 1);
        auto add = [&](float am, int m) {
          const float4 x = *reinterpret_cast<const float4*>(&cur[now][m][jl]);
          acc[0] = fmaf(am, x.x, acc[0]);
          acc[1] = fmaf(am, x.y, acc[1]);
          acc[2] = fmaf(am, x.z, acc[2]);
          acc[3] = fmaf(am, x.w, acc[3]);
        };
        if constexpr (!WIDE) {
          const float* src = row_of(p) + dv;
#pragma unroll 4
          for (int m = 0; m < dk; ++m) add(src[m], m);
        } else
#pragma unroll 1
        for (int stretch = 0; stretch < STRETCHES; ++stretch) {
          float4 have[NB];
#pragma unroll
          for (int q = 0; q < NB; ++q) have[q] = a[q];
          if (stretch + 1 < STRETCHES) request_a(p, stretch + 1);
          else if (p + 2 < n) request_a(p + 1, 0);
#pragma unroll
          for (int q = 0; q < NB; ++q) {
            const int m = (stretch * NB + q) * 4;
            add(have[q].x, m);
            add(have[q].y, m + 1);
            add(have[q].z, m + 2);
            add(have[q].w, m + 3);
          }
        }
      } else {
        const float k = keep;
        if (p + 2 < n) request_b(p + 1);
        acc[0] = fmaf(k, mine.x, acc[0]);
        acc[1] = fmaf(k, mine.y, acc[1]);
        acc[2] = fmaf(k, mine.z, acc[2]);
        acc[3] = fmaf(k, mine.w, acc[3]);
      }
      if (i < dk) *reinterpret_cast<float4*>(&cur[now ^ 1][i][jl]) = float4{acc[0], acc[1], acc[2], acc[3]};
    }
    if (i < dk) {      // (a lane reads and writes its own elements of B; A is only read)
      float* dst = row_of(p);
      const float v[4] = {mine.x, mine.y, mine.z, mine.w};
#pragma unroll
      for (int c = 0; c < 4; ++c)
        if (j0 + c < dv) dst[j0 + c] = v[c];
    }
    __syncthreads();
  }
}

template <int DKP, int G, int JPT, int TILE, bool DELTA>
void launch_state(StateArgs A, int S, hipStream_t s) {
  constexpr int CB = JPT * 256 / G;
  if (A.piece == 0) {
    A.pieces_per_seq = 1;
    A.col_blocks = (A.dv + CB - 1) / CB;
    gated_state_kernel<DKP, G, JPT, TILE, DELTA, false><<<dim3(A.heads * A.col_blocks, S), 256, 0, s>>>(A);
    return;
  }
  const int W = DELTA ? A.dv + A.dk : A.dv;
  StateArgs E = A;
  E.col_blocks = (W + CB - 1) / CB;
  gated_state_kernel<DKP, G, JPT, TILE, DELTA, true><<<dim3(E.heads * E.col_blocks, S * A.pieces_per_seq), 256, 0, s>>>(E);
  E.col_blocks = (A.dv + kPassCols - 1) / kPassCols;
  constexpr int PK = DKP < 64 ? 64 : DKP;
  const dim3 grid(E.heads * E.col_blocks, S);
  if (!DELTA || (A.dk % 4 == 0 && A.dv % 4 == 0)) gated_state_pass_kernel<PK, DELTA, true><<<grid, PK * 4, 0, s>>>(E);
  else gated_state_pass_kernel<PK, DELTA, false><<<grid, PK * 4, 0, s>>>(E);
  E.col_blocks = (A.dv + CB - 1) / CB;
  gated_state_kernel<DKP, G, JPT, TILE, DELTA, false><<<dim3(E.heads * E.col_blocks, S * A.pieces_per_seq), 256, 0, s>>>(E);
}

}  // namespace kvcm

using namespace kvcm;

extern "C" {

// floats of scratch for a step of `rows` rows and S sequences walked in pieces
long long kvcm_gated_state_carry_floats(int rows, int S, int heads, int dk, int dv, int delta, int piece) {
  if (piece <= 0 || rows < 0 || S < 0) return 0;
  const long long places = rows / piece + S + 1;
  return places * heads * (static_cast<long long>(dk) * (delta ? dv + dk : dv) + 1);
}

// q, k [T, groups*dk], v [T, heads*dv], a (and with delta b) [T, heads] at their own strides; dt_bias, a_log (and without delta
// d_skip) [heads]; decay [heads] (delta 0): a fixed decay in their place; silu_in (with decay): q, k and v are silu of what is
// given; o [T, >= heads*dv]; state [slots, heads, dk, dv]; all 32-bit.  piece > 0: runs (max_run: the longest) are
// walked in pieces of that many rows, with `carry` as scratch.
int kvcm_gated_state(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* a, int lda, const float* b,
                     int ldb, const float* dt_bias, const float* a_log, const float* d_skip, const float* decay, int silu_in, int delta, float* o, int ldo, float* state,
                     const int* run_start, const int* seq_start, const int* state_slots, int S, int heads, int groups, int dk, int dv,
                     int T, int piece, int max_run, float* carry, long long carry_floats, hipStream_t s) {
  if (S == 0 || T == 0) return 0;
  KVCM_REQUIRE(S > 0 && T > 0 && heads > 0 && groups > 0 && dk > 0 && dv > 0, "gated_state: bad sizes S=%d heads=%d dk=%d dv=%d", S, heads, dk, dv);
  KVCM_REQUIRE(heads % groups == 0, "gated_state: %d heads are not a multiple of %d groups", heads, groups);
  KVCM_REQUIRE(dk <= 256, "gated_state: a key size of %d is not supported (up to 256)", dk);
  KVCM_REQUIRE(ldq >= groups * dk && ldk >= groups * dk && ldv >= heads * dv && (decay || lda >= heads) && (!delta || ldb >= heads) && ldo >= heads * dv,
               "gated_state: row strides too small");
  KVCM_REQUIRE(q && k && v && o && state && (decay || (a && dt_bias && a_log && (delta ? b != nullptr : d_skip != nullptr))), "gated_state: an operand is missing");
  KVCM_REQUIRE(!(decay && delta) && (decay || !silu_in), "gated_state: a fixed decay beside the delta rule, or silu without one, is not supported");
  KVCM_REQUIRE(static_cast<long long>(heads) * ((dv + dk + 15) / 16) < (1ll << 31), "gated_state: too many heads");
  StateArgs A = {q, k, v, a, b, ldq, ldk, ldv, lda, ldb, dt_bias, a_log, d_skip, decay, silu_in, o, ldo, state, run_start, seq_start, state_slots,
                 heads, groups, dk, dv, 0, carry, piece, 1, 0};
  if (piece > 0) {
    KVCM_REQUIRE(max_run > 0 && carry && carry_floats >= kvcm_gated_state_carry_floats(T, S, heads, dk, dv, delta, piece),
                 "gated_state: the scratch for the pieces is too small");
    A.pieces_per_seq = (max_run + piece - 1) / piece;
    A.total_pieces = T / piece + S + 1;
  }
  KVCM_REQUIRE(static_cast<long long>(S) * A.pieces_per_seq <= 65535, "gated_state: too many sequences and pieces for one launch");
#define KVCM_STATE(DKP, G, JPT, TILE)                               \
  {                                                                 \
    if (delta) launch_state<DKP, G, JPT, TILE, true>(A, S, s);      \
    else launch_state<DKP, G, JPT, TILE, false>(A, S, s);           \
  }
  // steps of single rows spread a state over as many workgroups as they can; runs of rows give a lane more of it to keep
  const bool rows = max_run >= 16;
  if (dk <= 16) KVCM_STATE(16, 4, 1, 8)
  else if (dk <= 32) KVCM_STATE(32, 8, 1, 8)
  else if (dk <= 64) { if (rows) KVCM_STATE(64, 4, 1, 8) else KVCM_STATE(64, 8, 1, 8) }
  else if (dk <= 128) { if (rows) KVCM_STATE(128, 8, 2, 8) else KVCM_STATE(128, 16, 1, 8) }
  else KVCM_STATE(256, 16, 1, 4)
#undef KVCM_STATE
  return launch_status("gated_state");
}

}  // extern "C"
